// delta.hip - the gated delta rule with a decay per head and key channel, with its short convolutions, norms and gates.
//   S <- g * S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q          S [dim, vdim] per head, float32
// Kernels:
//  * delta_decode_kernel: one token per sequence, everything of a (sequence, head) in one workgroup: convolutions from the ring of
//    earlier inputs, unit norms, the low-rank decay and gate products, the state update (state in registers between its two passes) and the
//    normed, gated read-out.  One launch instead of five, the state is read and written once.
//  * delta_lowrank_kernel, delta_prep_*_kernel, delta_chunk_kernel / delta_scan_kernel / delta_out_kernel: several tokens per sequence.  The first do
//    what is parallel over tokens or chunks of 16 tokens; scan passes the state from chunk to chunk on the float32 matrix pipe; out norms and gates.
// The ring of convolution inputs is indexed by position modulo taps: the current token's entry is never one that the same step reads, so
// heads that share a q / k head need no ordering, and a sequence that starts over in a used slot reads none of the old entries.
#include "common.h"

namespace chatts {

// ---- one token per sequence -----------------------------------------------------------------------------------------------------
// thread (tx, ty): 4 consecutive value columns tx * 4, key rows ty + TY * r.
// Everything a workgroup reads is requested at once, the small inputs first (loads return in order) and the state last, so that the convolutions,
// norms and gates are formed while the state is on its way.  No load is conditional: addresses are clamped and the values selected.
template <int NT, int NR, int NU>      // NU: channels of q, k, v per thread
__global__ __launch_bounds__(NT) void delta_decode_kernel(ChattsDeltaArgs p, int TX) {
  extern __shared__ float sm[];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
  const int pos = p.rows[row].pos, slot = p.rows[row].slot;
  if (pos < 0) return;
  const int dim = p.dim, vdim = p.vdim, v4 = (vdim + 3) & ~3;
  const int group = p.heads / p.kv_heads, hk = h / group;
  float* red = sm;                      // NT * 4
  float* su = red + NT * 4;             // (red and su are read as float4)
  float* sv = su + v4;
  float* sgate = sv + v4;
  float* sq = sgate + v4;
  float* sk = sq + dim;
  float* sg = sk + dim;
  float* sa = sg + dim;
  float* sgi = sa + p.rank_a;
  float* scratch = sgi + p.rank_g;      // NT / 64
  const int tx = tid & (TX - 1), ty = tid / TX, TY = NT / TX;
  const bool live = tx * 4 < v4;
  float* S = p.state + ((size_t)slot * p.heads + h) * dim * v4;
  const int stride = TY * v4;
  float* Sp = S + (size_t)ty * v4 + tx * 4;
  const float* pr = p.proj + (size_t)row * p.ld_proj;
  float* ring = p.ring + (size_t)slot * p.taps * p.conv_ch;
  const int total = 2 * dim + vdim;
  auto channel = [&](int i) {
    if (i < dim) return p.off_q + hk * dim + i;
    if (i < 2 * dim) return p.off_k + hk * dim + i - dim;
    return p.off_v + h * vdim + i - 2 * dim;
  };
  constexpr int kPast = 3;      // earlier tokens requested ahead; more taps take the loop below
  float cur[NU], past[NU][kPast], cw[NU][kPast + 1];
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int i = u * NT + tid, ch = channel(i < total ? i : total - 1);
    cur[u] = pr[ch];
    cw[u][0] = p.conv_w[(size_t)(p.taps - 1) * p.conv_ch + ch];
#pragma unroll
    for (int g = 1; g <= kPast; ++g) {
      const bool ok = g < p.taps && pos >= g;
      past[u][g - 1] = ring[(size_t)((ok ? pos - g : pos) % p.taps) * p.conv_ch + ch];
      cw[u][g] = p.conv_w[(size_t)(g < p.taps ? p.taps - 1 - g : 0) * p.conv_ch + ch];
      if (!ok) cw[u][g] = 0.f;
    }
  }
  const float beta_in = pr[p.off_b + h];
  constexpr int kW = 8;      // 8-value pieces of this thread's low-rank row requested ahead
  const bool dec = tid < dim;
  const int lr = tid < dim + vdim ? tid : dim + vdim - 1, lrow = dec ? h * dim + tid : h * vdim + (lr - dim < 0 ? 0 : lr - dim);
  const int lrank = (dec ? p.rank_a : p.rank_g) >> 3, lrows = dec ? p.heads * dim : p.heads * vdim;
  const uint16_t* lw = (dec ? p.a2d : p.g2d) + (size_t)lrow * 8;
  u32x4 wv[kW];
#pragma unroll
  for (int c = 0; c < kW; ++c) wv[c] = *reinterpret_cast<const u32x4*>(lw + (size_t)(c < lrank ? c : 0) * lrows * 8);
  const float lbias = dec ? p.dt_bias[lrow] : 0.f, lneg = dec ? p.neg_a[lrow] : 0.f;
  const float a_in = pr[p.off_a + (tid < p.rank_a ? tid : 0)], g_in = pr[p.off_g + (tid < p.rank_g ? tid : 0)];
  f32x4 s[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int i = ty + TY * r < dim ? ty + TY * r : dim - 1;
    s[r] = *reinterpret_cast<const f32x4*>(S + (size_t)i * v4 + (live ? tx * 4 : 0));
  }
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int i = u * NT + tid;
    if (i >= total) continue;
    const int ch = channel(i);
    float acc = 0.f;
    for (int g = p.taps - 1; g > kPast; --g)
      if (pos >= g) acc += p.conv_w[(size_t)(p.taps - 1 - g) * p.conv_ch + ch] * ring[(size_t)((pos - g) % p.taps) * p.conv_ch + ch];
#pragma unroll
    for (int g = kPast; g >= 1; --g)
      if (cw[u][g] != 0.f) acc += cw[u][g] * past[u][g - 1];      // (an unused entry may hold anything)
    acc += cw[u][0] * cur[u];
    if (i >= 2 * dim || h == hk * group) ring[(size_t)(pos % p.taps) * p.conv_ch + ch] = cur[u];      // q / k: the first head of the group
    acc *= sigmoid_f(acc);
    if (i < dim) sq[i] = acc;
    else if (i < 2 * dim) sk[i - dim] = acc;
    else sv[i - 2 * dim] = acc;
  }
  if (tid < p.rank_a) sa[tid] = a_in;
  if (tid < p.rank_g) sgi[tid] = g_in;
  for (int i = tid + NT; i < p.rank_a; i += NT) sa[i] = pr[p.off_a + i];
  for (int i = tid + NT; i < p.rank_g; i += NT) sgi[i] = pr[p.off_g + i];
  __syncthreads();
  float qs = 0.f, ks = 0.f;      // every wave forms both norms
  for (int i = tid & 63; i < dim; i += 64) { qs += sq[i] * sq[i]; ks += sk[i] * sk[i]; }
  qs = wave_sum(qs);
  ks = wave_sum(ks);
  const float qn = rsqrtf((float)dim) / sqrtf(qs + 1e-6f), kn = 1.0f / sqrtf(ks + 1e-6f);
  auto dot8 = [](const u32x4& w, const float* x, float acc) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      acc += bf16_lo(w[j]) * x[2 * j];
      acc += bf16_hi(w[j]) * x[2 * j + 1];
    }
    return acc;
  };
  for (int i = tid; i < dim + vdim; i += NT) {
    const bool de = i < dim;
    const int o = de ? h * dim + i : h * vdim + i - dim, rank8 = (de ? p.rank_a : p.rank_g) >> 3, rows = de ? p.heads * dim : p.heads * vdim;
    const uint16_t* w = (de ? p.a2d : p.g2d) + (size_t)o * 8;
    const float* x = de ? sa : sgi;
    float acc = 0.f;
    int c = 0;
    if (i == tid) {
#pragma unroll
      for (int e = 0; e < kW; ++e)
        if (e < rank8) acc = dot8(wv[e], x + e * 8, acc);
      c = kW;
    }
    for (; c < rank8; ++c) acc = dot8(*reinterpret_cast<const u32x4*>(w + (size_t)c * rows * 8), x + c * 8, acc);
    if (de) sg[i] = exp_hw((i == tid ? lneg : p.neg_a[o]) * softplus_f(acc + (i == tid ? lbias : p.dt_bias[o])));
    else sgate[i - dim] = sigmoid_f(acc);
  }
#pragma unroll
  for (int r = 0; r < NR; ++r)
    if (!(pos > 0 && live && ty + TY * r < dim)) s[r] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const float beta = sigmoid_f(beta_in);
  __syncthreads();
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int i = ty + TY * r;
    if (i < dim) {
      const float g = sg[i], k = sk[i] * kn;
#pragma unroll
      for (int j = 0; j < 4; ++j) { s[r][j] *= g; acc[j] += s[r][j] * k; }
    }
  }
  *reinterpret_cast<f32x4*>(red + tid * 4) = acc;
  __syncthreads();
  for (int j = tid; j < v4; j += NT) {
    float t = 0.f;
    for (int y = 0; y < TY; ++y) t += red[(y * TX + (j >> 2)) * 4 + (j & 3)];
    su[j] = j < vdim ? beta * (sv[j] - t) : 0.f;
  }
  __syncthreads();
  acc = (f32x4){0.f, 0.f, 0.f, 0.f};
  if (live) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(su + tx * 4);
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const int i = ty + TY * r;
      if (i < dim) {
        const float k = sk[i] * kn, q = sq[i] * qn;
#pragma unroll
        for (int j = 0; j < 4; ++j) { s[r][j] += k * u[j]; acc[j] += s[r][j] * q; }
        *reinterpret_cast<f32x4*>(Sp + (size_t)r * stride) = s[r];
      }
    }
  }
  *reinterpret_cast<f32x4*>(red + tid * 4) = acc;
  __syncthreads();
  float o = 0.f;
  if (tid < vdim)
    for (int y = 0; y < TY; ++y) o += red[(y * TX + (tid >> 2)) * 4 + (tid & 3)];
  const float ss = block_sum<NT / 64>(tid < vdim ? o * o : 0.f, scratch);
  if (tid < vdim)
    store_operand(p.out, row, h * vdim + tid, o * (1.0f / sqrtf(ss / (float)vdim + p.eps)) * p.norm_w[tid] * sgate[tid]);
}

// ---- several tokens: what is parallel over tokens -------------------------------------------------------------------------------
// convolution + silu of channel ch for rows row0 .. row0 + ROWS: the window slides in registers.  Tokens before a row's segment come from the ring.
template <int TAPS, int ROWS>      // TAPS 0: any number of taps
__device__ __forceinline__ void conv_rows(const ChattsDeltaArgs& p, int row0, const ChattsRow (&R)[ROWS], int ch, float (&y)[ROWS]) {
  if constexpr (TAPS > 0) {
    float x[ROWS + TAPS - 1], w[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = p.conv_w[(size_t)j * p.conv_ch + ch];
#pragma unroll
    for (int j = 0; j < ROWS + TAPS - 1; ++j) {
      int r = row0 + j - (TAPS - 1);
      r = r < 0 ? 0 : (r > p.n_rows - 1 ? p.n_rows - 1 : r);
      x[j] = p.proj[(size_t)r * p.ld_proj + ch];
    }
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const int lag = TAPS - 1 - j;
        float v = x[i + j];
        if (row0 + i - lag < R[i].first) {      // (uniform over the wave)
          const int q = R[i].pos - lag;
          v = q < 0 ? 0.f : p.ring[((size_t)R[i].slot * TAPS + q % TAPS) * p.conv_ch + ch];
        }
        acc += w[j] * v;
      }
      y[i] = acc * sigmoid_f(acc);
    }
  } else {
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      float acc = 0.f;
      for (int j = 0; j < p.taps; ++j) {
        const int lag = p.taps - 1 - j, q = R[i].pos - lag, r = row0 + i - lag;
        if (q < 0) continue;
        acc += p.conv_w[(size_t)j * p.conv_ch + ch] * (r >= R[i].first ? p.proj[(size_t)r * p.ld_proj + ch]
                                                                       : p.ring[((size_t)R[i].slot * p.taps + q % p.taps) * p.conv_ch + ch]);
      }
      y[i] = acc * sigmoid_f(acc);
    }
  }
}
template <int ROWS>
__device__ __forceinline__ void prep_rows(const ChattsDeltaArgs& p, int row0, ChattsRow (&R)[ROWS], bool (&live)[ROWS]) {
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int r = row0 + i < p.n_rows ? row0 + i : p.n_rows - 1;
    R[i] = p.rows[r];
    live[i] = row0 + i < p.n_rows && R[i].pos >= 0;
    if (!live[i]) R[i] = ChattsRow{0, 0, r, 0};
  }
}

// q / k heads: a wave = one head of four rows
constexpr int kQkRows = 4, kVRows = 8;
template <int TAPS, int NCH>      // NCH: 64-channel pieces of a head
__global__ __launch_bounds__(256) void delta_prep_qk_kernel(ChattsDeltaArgs p) {
  const int row0 = blockIdx.x * kQkRows, lane = threadIdx.x & 63, e = blockIdx.y * 4 + (threadIdx.x >> 6), dim = p.dim;
  if (e >= p.kv_heads) return;
  ChattsRow R[kQkRows];
  bool live[kQkRows];
  prep_rows(p, row0, R, live);
  float q[NCH][kQkRows], k[NCH][kQkRows], qs[kQkRows], ks[kQkRows];
#pragma unroll
  for (int i = 0; i < kQkRows; ++i) qs[i] = ks[i] = 0.f;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int ch = c * 64 + lane;
    const bool ok = ch < dim;
    conv_rows<TAPS>(p, row0, R, p.off_q + e * dim + (ok ? ch : 0), q[c]);
    conv_rows<TAPS>(p, row0, R, p.off_k + e * dim + (ok ? ch : 0), k[c]);
#pragma unroll
    for (int i = 0; i < kQkRows; ++i) {
      if (!ok) q[c][i] = k[c][i] = 0.f;
      qs[i] += q[c][i] * q[c][i];
      ks[i] += k[c][i] * k[c][i];
    }
  }
  const float qscale = rsqrtf((float)dim);
#pragma unroll
  for (int i = 0; i < kQkRows; ++i) {
    const float fq = qscale / sqrtf(wave_sum(qs[i]) + 1e-6f), fk = 1.0f / sqrtf(wave_sum(ks[i]) + 1e-6f);
    if (!live[i]) continue;
    const size_t at = (size_t)(row0 + i) * p.kv_heads + e;
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int ch = c * 64 + lane;
      if (ch < dim) {
        p.q[at * dim + ch] = q[c][i] * fq;
        p.k[at * dim + ch] = k[c][i] * fk;
      }
    }
  }
}

// v and beta: a wave = 64 channels of eight rows
template <int TAPS>
__global__ __launch_bounds__(256) void delta_prep_v_kernel(ChattsDeltaArgs p) {
  const int row0 = blockIdx.x * kVRows, lane = threadIdx.x & 63, e = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int nv = p.heads * p.vdim, vchunks = (nv + 63) / 64;
  ChattsRow R[kVRows];
  bool live[kVRows];
  prep_rows(p, row0, R, live);
  if (e < vchunks) {
    const int ch = e * 64 + lane;
    if (ch >= nv) return;
    float y[kVRows];
    conv_rows<TAPS>(p, row0, R, p.off_v + ch, y);
#pragma unroll
    for (int i = 0; i < kVRows; ++i)
      if (live[i]) p.v[(size_t)(row0 + i) * nv + ch] = y[i];
    return;
  }
  const int h = (e - vchunks) * 64 + lane;
  if (h < p.heads)
#pragma unroll
    for (int i = 0; i < kVRows; ++i)
      if (live[i]) p.beta[(size_t)(row0 + i) * p.heads + h] = sigmoid_f(p.proj[(size_t)(row0 + i) * p.ld_proj + p.off_b + h]);
}

// The low-rank products with what follows them:  g = exp(neg_a * softplus(A2 a + dt_bias)),  gate = sigmoid(G2 gin).  grid (row tiles of 16, blocks of
// 512 outputs): a wave keeps its 16 rows of a (or gin) in registers, split into bf16 planes (three of them in 32-bit runs: exact), and walks 8
// tiles of 16 outputs, the weights requested two tiles ahead.
constexpr int kLrTiles = 8;
template <int NP, int KMAX>      // planes, rank / 32
__global__ __launch_bounds__(256) void delta_lowrank_kernel(ChattsDeltaArgs p, int ablocks) {
  typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
  const bool dec = (int)blockIdx.y < ablocks;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, fr = lane & 15, fg = lane >> 4, m0 = blockIdx.x * 16;
  const int n = dec ? p.heads * p.dim : p.heads * p.vdim, rank = dec ? p.rank_a : p.rank_g, ldw = dec ? p.ld_a2 : p.ld_g2;
  const int n0 = (dec ? blockIdx.y : blockIdx.y - ablocks) * (64 * kLrTiles) + wave * (16 * kLrTiles);
  if (n0 >= n) return;
  const uint16_t* w = dec ? p.a2 : p.g2;
  const int r = m0 + fr < p.n_rows ? m0 + fr : p.n_rows - 1;
  const float* x = p.proj + (size_t)r * p.ld_proj + (dec ? p.off_a : p.off_g) + fg * 8;
  f32x4 acc[kLrTiles];
#pragma unroll
  for (int t = 0; t < kLrTiles; ++t) acc[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < rank; k0 += 32 * KMAX) {
    bf16x8_t a[KMAX][NP];
    int ko[KMAX];      // K offsets; past the rank: offset 0 and zeros in a
#pragma unroll
    for (int k = 0; k < KMAX; ++k) {
      const bool ok = k0 + k * 32 < rank;
      ko[k] = ok ? k0 + k * 32 : 0;
      const f32x4 x0 = *reinterpret_cast<const f32x4*>(x + ko[k]), x1 = *reinterpret_cast<const f32x4*>(x + ko[k] + 4);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float v = ok ? (j < 4 ? x0[j] : x1[j - 4]) : 0.f;
#pragma unroll
        for (int q = 0; q < NP; ++q) {
          a[k][q][j] = (__bf16)v;
          v -= (float)a[k][q][j];
        }
      }
    }
    bf16x8_t b[3][KMAX];
    auto request = [&](int t, bf16x8_t (&dst)[KMAX]) __attribute__((always_inline)) {
      int o = n0 + t * 16 + fr;
      if (o > n - 1) o = n - 1;
#pragma unroll
      for (int k = 0; k < KMAX; ++k) dst[k] = *reinterpret_cast<const bf16x8_t*>(w + (size_t)o * ldw + ko[k] + fg * 8);
    };
    request(0, b[0]);
    request(1, b[1]);
#pragma unroll
    for (int t = 0; t < kLrTiles; ++t) {
      if (t + 2 < kLrTiles) request(t + 2, b[(t + 2) % 3]);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int k = 0; k < KMAX; ++k)
#pragma unroll
        for (int q = NP - 1; q >= 0; --q) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(b[t % 3][k], a[k][q], acc[t], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
  }
  // a lane: 4 consecutive outputs of row m0 + fr per tile
  const bool quads = (n & 3) == 0;
  f32x4 na[kLrTiles], bias[kLrTiles];
  if (dec)
#pragma unroll
    for (int t = 0; t < kLrTiles; ++t) {
      const int o0 = n0 + t * 16 + fg * 4;
      if (quads) {
        const int o = o0 < n ? o0 : 0;
        na[t] = *reinterpret_cast<const f32x4*>(p.neg_a + o);
        bias[t] = *reinterpret_cast<const f32x4*>(p.dt_bias + o);
      } else {
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int o = o0 + q < n ? o0 + q : n - 1;
          na[t][q] = p.neg_a[o];
          bias[t][q] = p.dt_bias[o];
        }
      }
    }
  // ... turned round in LDS (a wave's own part), so that a row's outputs leave as whole cache lines
  constexpr int kCols = 16 * kLrTiles, kLd = kCols + 4;
  __shared__ __attribute__((aligned(16))) float turn[4][16][kLd];
#pragma unroll
  for (int t = 0; t < kLrTiles; ++t) {
    f32x4 v;
#pragma unroll
    for (int q = 0; q < 4; ++q) v[q] = dec ? exp_hw(na[t][q] * softplus_f(acc[t][q] + bias[t][q])) : sigmoid_f(acc[t][q]);
    *reinterpret_cast<f32x4*>(&turn[wave][fr][t * 16 + fg * 4]) = v;
  }
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  constexpr int kLanes = kCols / 4, kRows = 64 / kLanes;      // lanes of a row, rows at a time
  float* dst = dec ? p.g : p.gate;
  const int o0 = n0 + (lane % kLanes) * 4;
#pragma unroll
  for (int i = 0; i < 16 / kRows; ++i) {
    const int rl = i * kRows + lane / kLanes, row = m0 + rl;
    const f32x4 v = *reinterpret_cast<const f32x4*>(&turn[wave][rl][(lane % kLanes) * 4]);
    if (row >= p.n_rows) continue;
    if (quads) {
      if (o0 < n) *reinterpret_cast<f32x4*>(dst + (size_t)row * n + o0) = v;
    } else {
#pragma unroll
      for (int q = 0; q < 4; ++q)
        if (o0 + q < n) dst[(size_t)row * n + o0 + q] = v[q];
    }
  }
}

template <int TAPS>
static void launch_prep(const ChattsDeltaArgs* a, hipStream_t s) {
  const dim3 g((a->n_rows + kQkRows - 1) / kQkRows, (a->kv_heads + 3) / 4), b(256);
  if (a->dim <= 64) hipLaunchKernelGGL((delta_prep_qk_kernel<TAPS, 1>), g, b, 0, s, *a);
  else if (a->dim <= 128) hipLaunchKernelGGL((delta_prep_qk_kernel<TAPS, 2>), g, b, 0, s, *a);
  else hipLaunchKernelGGL((delta_prep_qk_kernel<TAPS, 4>), g, b, 0, s, *a);
  const int items = (a->heads * a->vdim + 63) / 64 + (a->heads + 63) / 64;
  hipLaunchKernelGGL(delta_prep_v_kernel<TAPS>, dim3((a->n_rows + kVRows - 1) / kVRows, (items + 3) / 4), b, 0, s, *a);
}

// ---- the recurrence over a span, 16 tokens (a chunk) at a time -----------------------------------------------------------------------
// Within a chunk that starts from state S, with G_t = g_0 .. g_t (products per key channel, g of the chunk's tokens) and D(s, t) = g_{s+1} .. g_t:
//   u_t = beta_t (v_t - S^T (G_t k_t) - sum_{s < t} A_ts u_s),   A_ts = k_t . (D(s, t) k_s)
//   o_t = S^T (G_t q_t) + sum_{s <= t} P_ts u_s,                 P_ts = q_t . (D(s, t) k_s)
//   S  <- G_15 S + sum_s (D(s, 15) k_s) u_s^T
// Every decay product runs forward in time (factors <= 1, nothing is divided: strong decays vanish instead of overflowing).  With
// T = (I + diag(beta) A)^-1 diag(beta) the first line is u = T (v - S^T (G k)).  All of G k, G q, D(., 15) k, T, P and G_15 depend on the
// inputs only: delta_chunk_kernel forms them for all chunks in parallel; delta_scan_kernel is left with small products that pass the state
// along, on the float32 matrix pipe.  Rows past the end of a span count as k = q = 0, g = 1, beta = 0: they change nothing.
//
// A (chunk, head) holds, in floats, D = 64 NC channels:  G k [D / 16][64][4] | G q, the same | D(., 15) k [D / 16][64][4] | T [64][4] | P [64][4] | G_15 [D],
// each in the order in which the 64 lanes of a wave read matrix fragments.  Chunk c of span i is number row0 / 16 + i + c.
constexpr int kChunk = CHATTS_DELTA_CHUNK;
static_assert(kChunk == 16, "a chunk is a matrix fragment");
__host__ __device__ constexpr int chunk_floats(int nc) { return 64 * nc * (3 * kChunk + 1) + 512; }

template <int NC>
__global__ __launch_bounds__(256) void delta_chunk_kernel(ChattsDeltaArgs p) {
  constexpr int D = NC * 64, D4 = D / 4;
  __shared__ __attribute__((aligned(16))) float sk[kChunk][D], sq[kChunk][D], sg[kChunk][D];
  __shared__ float sa[kChunk][kChunk + 1], sb[kChunk];
  const int h = blockIdx.x, chunk = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int row = -1, n = 0;      // first row and rows of this chunk
  for (int i = 0; i < p.n_spans; ++i) {
    const int r0 = p.spans[i].row0, t = p.spans[i].t, c = chunk - (r0 / kChunk + i);
    if (c >= 0 && c * kChunk < t) { row = r0 + c * kChunk; n = t - c * kChunk; }
  }
  if (row < 0) return;
  if (n > kChunk) n = kChunk;
  const int dim = p.dim, hk = h / (p.heads / p.kv_heads), qrow = p.kv_heads * dim, grow = p.heads * dim;
  float* out = p.chunks + ((size_t)chunk * p.heads + h) * chunk_floats(NC);
#pragma unroll
  for (int e = 0; e < kChunk * D / 256; ++e) {
    const int j = e * 256 + tid, t = j / D, c = j % D;
    const bool ok = t < n && c < dim;
    const size_t r = row + (t < n ? t : 0);
    const int cc = c < dim ? c : 0;
    const float k = p.k[r * qrow + hk * dim + cc], q = p.q[r * qrow + hk * dim + cc], g = p.g[r * grow + h * dim + cc];
    sk[t][c] = ok ? k : 0.f;
    sq[t][c] = ok ? q : 0.f;
    sg[t][c] = ok ? g : 1.f;
  }
  if (tid < kChunk) sb[tid] = tid < n ? p.beta[(size_t)(row + tid) * p.heads + h] : 0.f;
  __syncthreads();
  {
    // A, P: thread = (token s, 1 / 16 of the channels), w = D(s, t) k_s walks forward in t
    const int s = tid >> 4, l16 = tid & 15;
    f32x4 w[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) w[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float ka = 0.f, kp = 0.f;      // of token t = l16
#pragma unroll 4
    for (int t = 0; t < kChunk; ++t) {
      float a = 0.f, b = 0.f;
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        const f32x4 g = *reinterpret_cast<const f32x4*>(&sg[t][c * 64 + l16 * 4]), k = *reinterpret_cast<const f32x4*>(&sk[t][c * 64 + l16 * 4]),
                    q = *reinterpret_cast<const f32x4*>(&sq[t][c * 64 + l16 * 4]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          w[c][j] = t == s ? k[j] : w[c][j] * g[j];
          a += k[j] * w[c][j];
          b += q[j] * w[c][j];
        }
      }
      a = row16_sum(a);
      b = row16_sum(b);
      ka = l16 == t ? a : ka;
      kp = l16 == t ? b : kp;
    }
    sa[l16][s] = l16 > s ? ka : 0.f;
    out[(3 * kChunk) * D + 256 + ((s >> 2) * 16 + l16) * 4 + (s & 3)] = l16 >= s ? kp : 0.f;      // P[t = l16][s]
  }
  // G k, G q and D(., 15) k of (token, 4 channels)
  constexpr int PER = D4 * kChunk / 256;
  f32x4 kt[PER];
#pragma unroll
  for (int e = 0; e < PER; ++e) {
    const int ct = e * 4 + wave, t = lane & 15, c = ct * 16 + (lane >> 4) * 4;
    f32x4 f = {1.f, 1.f, 1.f, 1.f}, b = {1.f, 1.f, 1.f, 1.f};
#pragma unroll
    for (int r = 0; r < kChunk; ++r) {
      const f32x4 g = *reinterpret_cast<const f32x4*>(&sg[r][c]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f[j] *= r <= t ? g[j] : 1.f;
        b[j] *= r > t ? g[j] : 1.f;
      }
    }
    const f32x4 k = *reinterpret_cast<const f32x4*>(&sk[t][c]), q = *reinterpret_cast<const f32x4*>(&sq[t][c]);
    f32x4 gk, gq;
#pragma unroll
    for (int j = 0; j < 4; ++j) { gk[j] = f[j] * k[j]; gq[j] = f[j] * q[j]; kt[e][j] = b[j] * k[j]; }
    *reinterpret_cast<f32x4*>(out + ct * 256 + lane * 4) = gk;
    *reinterpret_cast<f32x4*>(out + kChunk * D + ct * 256 + lane * 4) = gq;
    if (t == kChunk - 1) *reinterpret_cast<f32x4*>(out + 3 * kChunk * D + 512 + c) = f;
  }
  __syncthreads();      // (sg is free, sa complete)
#pragma unroll
  for (int e = 0; e < PER; ++e)
    *reinterpret_cast<f32x4*>(&sg[lane & 15][(e * 4 + wave) * 16 + (lane >> 4) * 4]) = kt[e];
  if (tid < kChunk) {      // column tid of T, by forward substitution
    float x[kChunk];
#pragma unroll
    for (int t = 0; t < kChunk; ++t) {
      float v = t == tid ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) v -= sa[t][s] * x[s];
      x[t] = sb[t] * v;
      out[(3 * kChunk) * D + ((tid >> 2) * 16 + t) * 4 + (tid & 3)] = x[t];
    }
  }
  __syncthreads();
#pragma unroll
  for (int e = 0; e < PER; ++e) {      // transposed: lane = (4 tokens lane >> 4, channel lane & 15)
    const int ct = e * 4 + wave;
    f32x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = sg[(lane >> 4) * 4 + j][ct * 16 + (lane & 15)];
    *reinterpret_cast<f32x4*>(out + 2 * kChunk * D + ct * 256 + lane * 4) = v;
  }
}

// grid (heads * column blocks of 16, spans), 4 waves: a wave holds NC tiles (16 channels x 16 columns) of the state as accumulators of the matrix
// pipe, which are also the right-hand operands of S^T (G k) and S^T (G q) - K slot g of product r means channel 4 g + r of a tile, token 4 g + r in
// the others, on both sides, so nothing is shuffled.  The waves' sums over channels meet in LDS once per chunk; u is formed by every wave.
template <int NC>
__global__ __launch_bounds__(256, NC <= 2 ? 2 : 1) void delta_scan_kernel(ChattsDeltaArgs p) {
  constexpr int D = NC * 64;
  __shared__ f32x4 sd[2][4][64];
  __shared__ float so[2][4][4][64];
  const ChattsSpan sp = p.spans[blockIdx.y];
  if (sp.t < 1) return;
  // (consecutive workgroups take consecutive heads: the column blocks of a head run on one XCD where heads % 8 == 0, its operands in that L2)
  const int cb = blockIdx.x / p.heads, h = blockIdx.x - cb * p.heads, tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const float mine[4] = {wave == 0 ? 1.f : 0.f, wave == 1 ? 1.f : 0.f, wave == 2 ? 1.f : 0.f, wave == 3 ? 1.f : 0.f};
  const int dim = p.dim, vdim = p.vdim, v4 = (vdim + 3) & ~3, fr = lane & 15, fg = lane >> 4, col = cb * 16 + fr;
  const bool live = col < vdim;
  float* S = p.state + ((size_t)sp.slot * p.heads + h) * dim * v4;
  f32x4 s[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = (wave * NC + c) * 16 + fg * 4 + r;
      s[c][r] = sp.pos0 > 0 && live && i < dim ? S[(size_t)i * v4 + col] : 0.f;
    }
  // addresses: a uniform base per chunk + constant 32-bit offsets of the lane
  const int vrow = p.heads * vdim, t_all = __builtin_amdgcn_readfirstlane(sp.t), row0 = __builtin_amdgcn_readfirstlane(sp.row0), nch = (t_all + kChunk - 1) / kChunk;
  const float* ops = p.chunks + ((size_t)(row0 / kChunk + blockIdx.y) * p.heads + h) * chunk_floats(NC);
  const size_t step = (size_t)p.heads * chunk_floats(NC);
  const float* gv = p.v + (size_t)row0 * vrow + h * vdim;
  float* go = p.o + (ptrdiff_t)row0 * vrow + h * vdim;
  const uint32_t lane16 = lane * 16, tile0 = wave * NC * 1024, gain0 = (wave * NC * 16 + fg * 4) * 4, p0 = lane16 + wave * 4;
  const uint32_t v_last = ((uint32_t)(t_all - 1) * vrow + (live ? col : 0)) * 4;
  uint32_t v_at[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) v_at[r] = ((uint32_t)(fg * 4 + r) * vrow + (live ? col : 0)) * 4;
  const uint32_t o_at = ((uint32_t)(fg * 4 + wave) * vrow + col) * 4;
  struct Ops { f32x4 k[NC], q[NC], kt[NC], g[NC], t, v; float pw; };
  auto at4 = [](const float* base, uint32_t off) __attribute__((always_inline)) { return *reinterpret_cast<const f32x4*>(reinterpret_cast<const char*>(base) + off); };
  auto at1 = [](const float* base, uint32_t off) __attribute__((always_inline)) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + off); };
  auto fetch_part = [&](int part, int c, Ops& o) __attribute__((always_inline)) {      // 0 .. kParts - 1
    if (c > nch - 1) c = nch - 1;
    const float* b = ops + (size_t)c * step;
    if (part == 0)
#pragma unroll
      for (int i = 0; i < NC; ++i) o.k[i] = at4(b + i * 256, tile0 + lane16);
    if (part == 1) {
      const uint32_t skip = (uint32_t)c * kChunk * vrow * 4;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const uint32_t off = v_at[r] + skip;
        o.v[r] = at1(gv, off < v_last ? off : v_last);
      }
    }
    if (part == 2) {
      o.t = at4(b + 3 * kChunk * D, lane16);
#pragma unroll
      for (int i = 0; i < NC; ++i) o.q[i] = at4(b + kChunk * D + i * 256, tile0 + lane16);
    }
    if (part == 3)
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        o.g[i] = at4(b + 3 * kChunk * D + 512 + i * 16, gain0);
        o.kt[i] = at4(b + 2 * kChunk * D + i * 256, tile0 + lane16);
      }
    if (part == 4) o.pw = at1(b + 3 * kChunk * D + 256, p0);
  };
  constexpr int kParts = 5;
  auto fetch = [&](int c, Ops& o) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < kParts; ++i) fetch_part(i, c, o);
  };
  f32x4 read_out = {0.f, 0.f, 0.f, 0.f};      // of the chunk before, this wave's channels and a quarter of its tokens' writes
  // this wave writes the tokens 4 g + wave of a chunk
  const int emit_from = live ? fg * 4 + wave : t_all;
  auto collect = [&](int b, float (&x)[4]) __attribute__((always_inline)) {
#pragma unroll
    for (int w = 0; w < 4; ++w) x[w] = so[b][w][wave][lane];
  };
  auto emit = [&](int c, const float (&x)[4]) __attribute__((always_inline)) {
    const int t0 = c * kChunk;
    if (c >= 0 && emit_from < t_all - t0) *reinterpret_cast<float*>(reinterpret_cast<char*>(go + (ptrdiff_t)t0 * vrow) + o_at) = (x[0] + x[1]) + (x[2] + x[3]);
  };
  auto hand_over = [&](int b) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < 4; ++r) so[b][wave][r][lane] = read_out[r];
  };
  auto meet = [&]() __attribute__((always_inline)) {
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
  };
  // S^T (G k) is the critical chain: it goes first; the products of S^T (G q) and the requests fill the waits of the exchange
  constexpr int kBefore = 3;
  auto chunk = [&](int c, Ops& o, Ops& later) __attribute__((always_inline)) {
    const int b = c & 1;
    f32x4 d = {0.f, 0.f, 0.f, 0.f}, e = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4 * NC; ++i) d = __builtin_amdgcn_mfma_f32_16x16x4f32(o.k[i >> 2][i & 3], s[i >> 2][i & 3], d, 0, 0, 0);
    hand_over(b);
    __builtin_amdgcn_sched_barrier(0);
    e = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[0][0], s[0][0], e, 0, 0, 0);
    __builtin_amdgcn_sched_barrier(0);
    sd[b][wave][lane] = d;
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int i = 1; i < kBefore; ++i) e = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i >> 2][i & 3], s[i >> 2][i & 3], e, 0, 0, 0);
    __builtin_amdgcn_sched_barrier(0);
    meet();
    const f32x4 d0 = sd[b][0][lane], d1 = sd[b][1][lane], d2 = sd[b][2][lane], d3 = sd[b][3][lane];
    float past[4];
    collect(b, past);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int i = kBefore; i < 4 * NC || i - kBefore < kParts; ++i) {      // requests for the chunk after the next go between products
      if (i < 4 * NC) e = __builtin_amdgcn_mfma_f32_16x16x4f32(o.q[i >> 2][i & 3], s[i >> 2][i & 3], e, 0, 0, 0);
      if (i - kBefore < kParts) fetch_part(i - kBefore, c + 2, later);
      __builtin_amdgcn_sched_barrier(0);
    }
    f32x4 u = {0.f, 0.f, 0.f, 0.f}, x;
#pragma unroll
    for (int r = 0; r < 4; ++r) x[r] = o.v[r] - ((d0[r] + d1[r]) + (d2[r] + d3[r]));
#pragma unroll
    for (int r = 0; r < 4; ++r) u = __builtin_amdgcn_mfma_f32_16x16x4f32(o.t[r], x[r], u, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NC; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[i][r] *= o.g[i][r];
    emit(c - 1, past);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < NC; ++i) s[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kt[i][r], u[r], s[i], 0, 0, 0);
    const float uw = u[0] * mine[0] + u[1] * mine[1] + u[2] * mine[2] + u[3] * mine[3];      // = u[wave], without branches
    read_out = __builtin_amdgcn_mfma_f32_16x16x4f32(o.pw, uw, e, 0, 0, 0);
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
  hand_over(nch & 1);
  meet();
  float past[4];
  collect(nch & 1, past);
  emit(nch - 1, past);
  if (live)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = (wave * NC + c) * 16 + fg * 4 + r;
        if (i < dim) S[(size_t)i * v4 + col] = s[c][r];
      }
}

// ---- norm + gate of the read-outs; the last `taps` rows of a span enter the ring (prep has read the old entries by now) -----------
// A head belongs to G lanes (a power of two, 4 G >= vdim), 4 consecutive columns each.
template <bool QUADS>      // vdim % 4 == 0
__global__ __launch_bounds__(256) void delta_out_kernel(ChattsDeltaArgs p, int G) {
  const int row = blockIdx.x, tid = threadIdx.x, per = 256 / G, i = (tid & (G - 1)) * 4;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const int vdim = p.vdim, vrow = p.heads * vdim;
  const float* o = p.o + (size_t)row * vrow;
  const float* gate = p.gate + (size_t)row * vrow;
  float w[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) w[j] = i + j < vdim ? p.norm_w[i + j] : 0.f;
  for (int h = blockIdx.y * per + tid / G; h < p.heads; h += gridDim.y * per) {      // (h is the same in all lanes of a group)
    float v[4] = {0.f, 0.f, 0.f, 0.f}, g[4] = {0.f, 0.f, 0.f, 0.f};
    const int at = h * vdim + i;
    if (QUADS) {
      if (i < vdim) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(o + at), y = *reinterpret_cast<const f32x4*>(gate + at);
#pragma unroll
        for (int j = 0; j < 4; ++j) { v[j] = x[j]; g[j] = y[j]; }
      }
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < vdim) { v[j] = o[at + j]; g[j] = gate[at + j]; }
    }
    float ss = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
    for (int x = 1; x < G; x <<= 1) ss += __shfl_xor(ss, x, 64);
    const float f = 1.0f / sqrtf(ss / (float)vdim + p.eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = v[j] * f * w[j] * g[j];
    if (QUADS) {
      if (i < vdim) store_operand4(p.out, row, at, v);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < vdim) store_operand(p.out, row, at + j, v[j]);
    }
  }
  if (R.rest < p.taps) {
    float* ring = p.ring + ((size_t)R.slot * p.taps + R.pos % p.taps) * p.conv_ch;
    for (int c = blockIdx.y * 256 + tid; c < p.conv_ch; c += gridDim.y * 256) ring[c] = p.proj[(size_t)row * p.ld_proj + c];
  }
}

static int check_delta(const ChattsDeltaArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->proj && a->rows && a->state && a->ring && a->conv_w && a->dt_bias && a->neg_a && a->norm_w, CHATTS_E_BADARG, "%s: null pointer", who);
  CHATTS_REQUIRE(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->taps >= 1, CHATTS_E_SHAPE, "%s: heads %d / %d, taps %d", who,
                 a->heads, a->kv_heads, a->taps);
  CHATTS_REQUIRE(a->dim >= 1 && a->dim <= 256 && a->vdim >= 1 && a->vdim <= 256, CHATTS_E_SHAPE, "%s: head sizes %d x %d (at most 256 x 256)", who,
                 a->dim, a->vdim);
  CHATTS_REQUIRE(a->rank_a % 8 == 0 && a->rank_g % 8 == 0 && a->ld_a2 % 8 == 0 && a->ld_g2 % 8 == 0, CHATTS_E_SHAPE, "%s: ranks must be multiples of 8", who);
  CHATTS_REQUIRE(a->ld_proj % 4 == 0 && a->conv_ch <= a->ld_proj && a->off_v + a->heads * a->vdim <= a->conv_ch &&
                     a->off_q + a->kv_heads * a->dim <= a->conv_ch && a->off_k + a->kv_heads * a->dim <= a->conv_ch, CHATTS_E_SHAPE, "%s: column blocks", who);
  return CHATTS_OK;
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_delta_decode(const ChattsDeltaArgs* a, chatts_stream_t stream) {
  if (const int rc = check_delta(a, "delta_decode")) return rc;
  CHATTS_REQUIRE(a->a2d && a->g2d && (a->out.f32 || a->out.hi) && a->out.ld >= a->heads * a->vdim, CHATTS_E_BADARG, "delta_decode: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  const int v4 = (a->vdim + 3) & ~3;
  int TX = 1;
  while (TX * 4 < v4) TX *= 2;
  auto rows_for = [&](int nt) { return (a->dim + nt / TX - 1) / (nt / TX); };
  const int nt = rows_for(256) > 32 ? 512 : 256, nr = rows_for(nt);
  const size_t lds = (size_t)(3 * a->dim + 3 * v4 + a->rank_a + a->rank_g + nt * 4 + 16 + 16) * sizeof(float);
  CHATTS_REQUIRE(lds <= 64 * 1024, CHATTS_E_SHAPE, "delta_decode: ranks %d / %d too large", a->rank_a, a->rank_g);
  const dim3 g(a->heads, a->n_rows);
  hipStream_t s = as_stream(stream);
  const int nu = (2 * a->dim + a->vdim + nt - 1) / nt;
#define CHATTS_DELTA_DECODE(NT, NR)                                                                                   \
  do {                                                                                                                 \
    if (nu <= 1) hipLaunchKernelGGL((delta_decode_kernel<NT, NR, 1>), g, dim3(NT), lds, s, *a, TX);                    \
    else if (nu == 2) hipLaunchKernelGGL((delta_decode_kernel<NT, NR, 2>), g, dim3(NT), lds, s, *a, TX);               \
    else hipLaunchKernelGGL((delta_decode_kernel<NT, NR, 3>), g, dim3(NT), lds, s, *a, TX);                            \
  } while (0)
  if (nt == 512) CHATTS_DELTA_DECODE(512, 32);
  else if (nr <= 4) CHATTS_DELTA_DECODE(256, 4);
  else if (nr <= 8) CHATTS_DELTA_DECODE(256, 8);
  else if (nr <= 16) CHATTS_DELTA_DECODE(256, 16);
  else CHATTS_DELTA_DECODE(256, 32);
#undef CHATTS_DELTA_DECODE
  CHATTS_CHECK_LAUNCH("delta_decode");
  return CHATTS_OK;
}

extern "C" int chatts_delta_prep(const ChattsDeltaArgs* a, chatts_stream_t stream) {
  if (const int rc = check_delta(a, "delta_prep")) return rc;
  CHATTS_REQUIRE(a->q && a->k && a->v && a->g && a->gate && a->beta && a->a2 && a->g2, CHATTS_E_BADARG, "delta_prep: null scratch");
  if (a->n_rows == 0) return CHATTS_OK;
  CHATTS_REQUIRE(a->rank_a % 32 == 0 && a->rank_g % 32 == 0 && ((uintptr_t)a->a2 % 16) == 0 && ((uintptr_t)a->g2 % 16) == 0 && a->off_a % 4 == 0 && a->off_g % 4 == 0 &&
                     ((uintptr_t)a->neg_a % 16) == 0 && ((uintptr_t)a->dt_bias % 16) == 0, CHATTS_E_SHAPE, "delta_prep: ranks %d / %d must be padded to multiples of 32", a->rank_a, a->rank_g);
  const int ablocks = (a->heads * a->dim + 64 * kLrTiles - 1) / (64 * kLrTiles), gblocks = (a->heads * a->vdim + 64 * kLrTiles - 1) / (64 * kLrTiles);
  const dim3 g((a->n_rows + 15) / 16, ablocks + gblocks), b(256);
  if (a->exact) hipLaunchKernelGGL((delta_lowrank_kernel<3, 4>), g, b, 0, as_stream(stream), *a, ablocks);
  else hipLaunchKernelGGL((delta_lowrank_kernel<2, 4>), g, b, 0, as_stream(stream), *a, ablocks);
  CHATTS_CHECK_LAUNCH("delta_lowrank");
  switch (a->taps) {
    case 2: launch_prep<2>(a, as_stream(stream)); break;
    case 3: launch_prep<3>(a, as_stream(stream)); break;
    case 4: launch_prep<4>(a, as_stream(stream)); break;
    default: launch_prep<0>(a, as_stream(stream)); break;
  }
  CHATTS_CHECK_LAUNCH("delta_prep");
  return CHATTS_OK;
}

extern "C" int64_t chatts_delta_chunk_floats(int heads, int dim, int n_rows, int n_spans) {
  return (int64_t)(n_rows / kChunk + n_spans) * heads * chunk_floats((dim + 63) / 64);
}

template <int NC>
static void launch_scan(const ChattsDeltaArgs* a, hipStream_t s) {
  hipLaunchKernelGGL(delta_chunk_kernel<NC>, dim3(a->heads, a->n_rows / kChunk + a->n_spans), dim3(256), 0, s, *a);
  hipLaunchKernelGGL(delta_scan_kernel<NC>, dim3(a->heads * ((a->vdim + 15) / 16), a->n_spans), dim3(256), 0, s, *a);
}

extern "C" int chatts_delta_scan(const ChattsDeltaArgs* a, chatts_stream_t stream) {
  if (const int rc = check_delta(a, "delta_scan")) return rc;
  CHATTS_REQUIRE(a->q && a->k && a->v && a->g && a->beta && a->chunks && a->o && a->spans, CHATTS_E_BADARG, "delta_scan: null scratch");
  CHATTS_REQUIRE(((uintptr_t)a->chunks % 16) == 0, CHATTS_E_SHAPE, "delta_scan: alignment");
  if (a->n_spans == 0) return CHATTS_OK;
  switch ((a->dim + 63) / 64) {
    case 1: launch_scan<1>(a, as_stream(stream)); break;
    case 2: launch_scan<2>(a, as_stream(stream)); break;
    case 3: launch_scan<3>(a, as_stream(stream)); break;
    default: launch_scan<4>(a, as_stream(stream)); break;
  }
  CHATTS_CHECK_LAUNCH("delta_scan");
  return CHATTS_OK;
}

extern "C" int chatts_delta_out(const ChattsDeltaArgs* a, chatts_stream_t stream) {
  if (const int rc = check_delta(a, "delta_out")) return rc;
  CHATTS_REQUIRE(a->o && a->gate && (a->out.f32 || a->out.hi) && a->out.ld >= a->heads * a->vdim, CHATTS_E_BADARG, "delta_out: null pointer");
  if (a->n_rows == 0) return CHATTS_OK;
  int lanes = 1;
  while (lanes * 4 < a->vdim) lanes *= 2;
  const int per = 256 / lanes;
  const dim3 g(a->n_rows, (a->heads + 2 * per - 1) / (2 * per));
  if (a->vdim % 4 == 0 && a->out.ld % 4 == 0) hipLaunchKernelGGL(delta_out_kernel<true>, g, dim3(256), 0, as_stream(stream), *a, lanes);
  else hipLaunchKernelGGL(delta_out_kernel<false>, g, dim3(256), 0, as_stream(stream), *a, lanes);
  CHATTS_CHECK_LAUNCH("delta_out");
  return CHATTS_OK;
}
