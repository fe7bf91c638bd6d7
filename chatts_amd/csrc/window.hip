// window.hip - attention over paged keys and values with grouped heads.  Optional, each by its own parameter: short convolutions, norms of queries and
// keys (per head, over all heads, unit after a rotation of pairs), mixed values; capped scores, a distance bias per head (linear or logarithmic), a sliding window that
// keeps a sequence's first tokens, chunks, a sink (one more term exp(0) in the denominator); an output gate per value or per head.
//   window_prep_kernel      per-head work: norms, rotation, values; queries as an operand, keys and values into their pages
//   window_prep_quads_kernel  the same, four channels a lane
//   window_prep_rows_kernel the same for layers with convolutions or norms over all heads: a workgroup owns whole rows
//   window_ring_kernel      the last convolution inputs of every segment
//   window_attend_kernel    one row and query head per workgroup, vector units: 32-bit runs, head sizes beyond the matrix kernels
//   window_decode_kernel    one row: the query heads of a key head share its tiles on the matrix pipe; tiles spread over waves and workgroups
//   window_prefill_kernel   flash attention for segments of many rows
// Pages: keys [page][kv head][token][dim_p], values [page][kv head][token][vdim_p]; a page holds a multiple of 64 tokens, so a tile of up to 64
// keys of a head is contiguous memory.
#include "gemm_common.h"

namespace chatts {

typedef short w16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) w16x4* lds_w16x4;

__device__ __forceinline__ size_t window_tile(const ChattsWindowArgs& p, int slot, int hk, int key) {      // row number of a key in its pool
  const int blk = p.table[(size_t)slot * p.table_stride + (key >> p.log_block)];
  return (((size_t)blk * p.kv_heads + hk) << p.log_block) + (key & ((1 << p.log_block) - 1));
}
__device__ __forceinline__ bool window_masked(const ChattsWindowArgs& p) { return p.window > 0 || p.chunk > 0; }
__device__ __forceinline__ int window_low(const ChattsWindowArgs& p, int pos) {      // first position that `pos` sees beside the kept ones
  if (p.window > 0) return pos - p.window + 1;
  return p.chunk > 0 ? pos - pos % p.chunk : 0;
}
// tiles of K keys that a row at `pos` (or rows pos_lo .. pos) sees: the first `kept`, then from `from` to the tile of pos
struct WindowTiles {
  int kept, from, last;
  __device__ __forceinline__ WindowTiles(const ChattsWindowArgs& p, int pos_lo, int pos, int log_tile) {
    last = pos >> log_tile;
    if (!window_masked(p)) { kept = 0; from = 0; return; }
    const int w = window_low(p, pos_lo);
    from = (w > 0 ? w : 0) >> log_tile;
    kept = (p.keep_first + (1 << log_tile) - 1) >> log_tile;
    if (kept > last + 1) kept = last + 1;
    if (from < kept) from = kept;
  }
  __device__ __forceinline__ int count() const { return kept + last + 1 - from; }
  __device__ __forceinline__ int tile(int i) const { return i < kept ? i : from + i - kept; }
};
__device__ __forceinline__ bool window_sees(const ChattsWindowArgs& p, int pos, int low, int key) { return key <= pos && (key >= low || key < p.keep_first); }
__device__ __forceinline__ float window_gate(const ChattsWindowArgs& p, size_t row, int h, int c) {
  return p.off_gate < 0 ? 1.f : sigmoid_f(p.proj[row * p.ld_proj + p.off_gate + (p.gate_heads ? h : h * p.vdim + c)]);
}
constexpr float kLog2e = 1.44269504088896341f;
// what the matrix kernels are compiled for (registers are scarce there): plain scores, a distance bias, capped scores (with chunks), a logarithmic bias, or
// whatever is set
enum { kPlain = 0, kSlope, kCap, kLog, kAny };
template <int SCORE>
__device__ __forceinline__ bool window_capped(const ChattsWindowArgs& p) { return SCORE == kCap || (SCORE == kAny && p.softcap > 0.f); }
template <int SCORE>
__device__ __forceinline__ bool window_sloped(const ChattsWindowArgs& p) { return SCORE == kSlope || (SCORE == kAny && p.slopes != nullptr); }
template <int SCORE>
__device__ __forceinline__ bool window_logged(const ChattsWindowArgs& p) { return SCORE == kLog || (SCORE == kAny && p.log_r1 != nullptr); }
// r1 log2(1 + r2 d)
__device__ __forceinline__ float window_log(float r1, float r2, float d) { return r1 * __builtin_amdgcn_logf(1.f + r2 * d); }
template <int SCORE>
__device__ __forceinline__ int window_low_of(const ChattsWindowArgs& p, int pos) {
  if (SCORE == kPlain || SCORE == kSlope || SCORE == kLog) return p.window > 0 ? pos - p.window + 1 : 0;      // (no chunks there)
  return window_low(p, pos);
}
// cap tanh(x / cap), in units of cap: tanh(y) = 1 - 2 / (1 + exp(2 y));  k = 2 log2(e) / cap
__device__ __forceinline__ float window_cap(float x, float k, float cap) { return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * k)); }

template <typename CT>
__device__ __forceinline__ CT to_page(float v) {
  if constexpr (sizeof(CT) == 4) return v;
  else return __builtin_bit_cast(uint16_t, (__bf16)v);
}

// grid (rows, n): the 4 n waves of a row take heads [q | k | v] in turn
template <typename CT>
__global__ __launch_bounds__(256) void window_prep_kernel(ChattsWindowArgs p) {
  const int row = blockIdx.x, lane = threadIdx.x & 63;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const int H = p.heads, G = p.kv_heads;
  const float* pr = p.proj + (size_t)row * p.ld_proj;
  for (int e = blockIdx.y * 4 + (threadIdx.x >> 6); e < H + 2 * G; e += 4 * gridDim.y) {
    const bool value = e >= H + G;
    const int hk = e < H ? 0 : (value ? e - H - G : e - H), n = value ? p.vdim : p.dim, np = value ? p.vdim_p : p.dim_p;
    const float* x = pr + (e < H ? p.off_q + e * p.dim : (value ? p.off_v + hk * p.vdim : p.off_k + hk * p.dim));
    float v[4], f = 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = j * 64 + lane < n ? x[j * 64 + lane] : 0.f;
    const float* w = value ? nullptr : (e < H ? p.q_norm : p.k_norm);
    auto inv_rms = [&]() { return 1.0f / sqrtf(wave_sum((v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3])) / (float)n + p.eps); };
    if (w) f = inv_rms();
    if (!value && (p.rot || p.unit)) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = j * 64 + lane;
        if (w) v[j] = c < n ? v[j] * f * w[c] : 0.f;
        if (j * 64 < p.rot) {      // (uniform; the other dimension of a pair is in the neighbouring lane)
          const float other = lane_xor1(v[j]);
          if (c < p.rot) {
            const size_t at = (size_t)R.pos * (p.rot >> 1) + (c >> 1);
            const float s = p.sin_tab[at];
            v[j] = v[j] * p.cos_tab[at] + (c & 1 ? other * s : -other * s);
          }
        }
      }
      f = p.unit ? inv_rms() : 1.f;
      w = nullptr;
    }
    if (value && p.vfirst) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = j * 64 + lane;
        if (c >= n) break;
        float* first = p.vfirst + (size_t)row * p.ld_vfirst + hk * n + c;
        if (p.vfirst_write) *first = v[j];
        else v[j] = (1.f - p.vmix) * v[j] + p.vmix * *first;
      }
    }
    CT* dst = nullptr;
    if (e >= H) dst = reinterpret_cast<CT*>(value ? p.vcache : p.kcache) + window_tile(p, R.slot, hk, R.pos) * np;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = j * 64 + lane;
      if (c >= np) break;
      const float y = v[j] * f * (w && c < n ? w[c] : 1.f);
      if (dst) dst[c] = to_page<CT>(y);
      else store_operand(p.q, row, e * p.dim_p + c, y);
    }
  }
}

// The same with quads of neighbouring channels per lane, LPH lanes to a head (dim, vdim <= 4 LPH, all sizes % 4 == 0): grid (rows, n), the 4 n waves of a row
// take 64 / LPH heads at a time, two such groups requested at once
template <int LPH>
__device__ __forceinline__ float head_sum(float v) {
  v = row16_sum(v);
  if (LPH >= 32) v += __shfl_xor(v, 16, 64);
  if (LPH >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}
__device__ __forceinline__ float quad_squares(const f32x4& v) { return (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }
template <typename CT>
__device__ __forceinline__ void store_page4(CT* dst, const f32x4& v) {
  if constexpr (sizeof(CT) == 4) *reinterpret_cast<f32x4*>(dst) = v;
  else *reinterpret_cast<w16x4*>(dst) = (w16x4){(short)to_page<CT>(v[0]), (short)to_page<CT>(v[1]), (short)to_page<CT>(v[2]), (short)to_page<CT>(v[3])};
}
template <typename CT, int LPH>
__global__ __launch_bounds__(256) void window_prep_quads_kernel(ChattsWindowArgs p) {
  constexpr int PER = 64 / LPH;
  const int row = blockIdx.x, lane = threadIdx.x & 63, H = p.heads, G = p.kv_heads, c = (lane & (LPH - 1)) * 4;
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const float* pr = p.proj + (size_t)row * p.ld_proj;
  const size_t page = window_tile(p, R.slot, 0, R.pos);      // head e of the page: e << log_block rows further
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  const int stride = 4 * PER * gridDim.y;
  for (int e0 = (blockIdx.y * 4 + (threadIdx.x >> 6)) * PER + lane / LPH; e0 - lane / LPH < H + 2 * G; e0 += 2 * stride) {      // (uniform)
    f32x4 x[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int e = e0 + u * stride;
      const bool value = e >= H + G;
      const int n = value ? p.vdim : p.dim;
      x[u] = zero;
      if (e < H + 2 * G && c < n) x[u] = *reinterpret_cast<const f32x4*>(pr + (e < H ? p.off_q + e * n : (value ? p.off_v + (e - H - G) * n : p.off_k + (e - H) * n)) + c);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int e = e0 + u * stride;
      const bool value = e >= H + G, live = e < H + 2 * G;
      const int n = value ? p.vdim : p.dim, np = value ? p.vdim_p : p.dim_p, hk = value ? e - H - G : e - H;
      f32x4 v = x[u];
      if (p.q_norm && !value) {
        const float* w = e < H ? p.q_norm : p.k_norm;
        const float f = 1.0f / sqrtf(head_sum<LPH>(quad_squares(v)) / (float)n + p.eps);
        if (c < n) v = v * f * *reinterpret_cast<const f32x4*>(w + c);
      }
      if (!value && c < p.rot) {
        const size_t at = (size_t)R.pos * (p.rot >> 1) + (c >> 1);
        const float c0 = p.cos_tab[at], s0 = p.sin_tab[at];
        v = (f32x4){v[0] * c0 - v[1] * s0, v[1] * c0 + v[0] * s0, v[2], v[3]};
        if (c + 2 < p.rot) {
          const float c1 = p.cos_tab[at + 1], s1 = p.sin_tab[at + 1];
          v = (f32x4){v[0], v[1], v[2] * c1 - v[3] * s1, v[3] * c1 + v[2] * s1};
        }
      }
      if (p.unit && !value) v = v * (1.0f / sqrtf(head_sum<LPH>(quad_squares(v)) / (float)n + p.eps));
      if (value && p.vfirst && live && c < n) {
        float* first = p.vfirst + (size_t)row * p.ld_vfirst + hk * n + c;
        if (p.vfirst_write) *reinterpret_cast<f32x4*>(first) = v;
        else v = (1.f - p.vmix) * v + p.vmix * *reinterpret_cast<const f32x4*>(first);
      }
      if (!live) continue;
      for (int cc = c; cc < np; cc += 4 * LPH) {      // (a second pass only over padding)
        const f32x4 y = cc == c ? v : zero;
        if (e < H) {
          const float o[4] = {y[0], y[1], y[2], y[3]};
          store_operand4(p.q, row, e * p.dim_p + cc, o);
        } else {
          store_page4(reinterpret_cast<CT*>(value ? p.vcache : p.kcache) + (page + ((size_t)hk << p.log_block)) * np + cc, y);
        }
      }
    }
  }
}

// A workgroup owns ROWS rows, a thread quads of channels of [q | k | v]: convolutions over a window of rows in registers (inputs before a segment come from
// the ring), norms over all heads, mixed values.
constexpr int kConvRegs = 4;      // taps whose weights stay in registers
template <typename CT, int NT, int NV, int ROWS>
__global__ __launch_bounds__(NT, 4) void window_prep_rows_kernel(ChattsWindowArgs p) {
  __shared__ float red[NT / 64][2 * ROWS];
  // neighbouring groups share rows: XCD x (= blockIdx % 8; speed only) takes a contiguous eighth of them
  const int share = gridDim.x >> 3, rem = gridDim.x & 7, xcd = blockIdx.x & 7;
  const int group = ROWS == 1 ? blockIdx.x : xcd * share + (xcd < rem ? xcd : rem) + (blockIdx.x >> 3);
  const int row0 = group * ROWS, tid = threadIdx.x, H = p.heads, G = p.kv_heads;
  const int n[3] = {H * p.dim, G * p.dim, G * p.vdim}, quads[3] = {(n[0] + 3) >> 2, (n[1] + 3) >> 2, (n[2] + 3) >> 2}, total = quads[0] + quads[1] + quads[2];
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  ChattsRow R[ROWS];
  size_t page[ROWS];
  bool one = true;      // the rows are consecutive rows of one segment
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    R[r] = row0 + r < p.n_rows ? p.rows[row0 + r] : ChattsRow{0, -1, 0, 0};
    page[r] = R[r].pos >= 0 ? window_tile(p, R[r].slot, 0, R[r].pos) : 0;
    one = one && R[r].pos >= 0 && R[r].first == R[0].first;
  }
  if (ROWS == 1 && R[0].pos < 0) return;
  auto place = [&](int u, int& block, int& c) __attribute__((always_inline)) {      // quad -> its block and first channel there
    block = u < quads[0] ? 0 : (u < quads[0] + quads[1] ? 1 : 2);
    c = 4 * (u - (block > 0 ? quads[0] : 0) - (block > 1 ? quads[1] : 0));
    return (block == 0 ? p.off_q : (block == 1 ? p.off_k : p.off_v)) + c;
  };
  auto input = [&](int r, int row, int back, int col) __attribute__((always_inline)) {      // the projected value `back` tokens before row r's
    if (row - back >= R[r].first) return *reinterpret_cast<const f32x4*>(p.proj + (size_t)(row - back) * p.ld_proj + col);
    const int q = R[r].pos - back;
    return q >= 0 ? *reinterpret_cast<const f32x4*>(p.ring + ((size_t)R[r].slot * p.taps + q % p.taps) * p.conv_ch + col) : zero;
  };
  f32x4 y[NV][ROWS];
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r = 0; r < ROWS; ++r) y[i][r] = zero;
  if (one && p.taps && p.taps <= kConvRegs && row0 - R[0].first >= p.taps - 1) {      // every input is a row of this step
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int u = i * NT + tid;
      if (u >= total) continue;
      int block, c;
      const int col = place(u, block, c);
      f32x4 w[kConvRegs], in[kConvRegs - 1 + ROWS];
#pragma unroll
      for (int j = 0; j < kConvRegs - 1 + ROWS; ++j)      // input j: row row0 + j - (kConvRegs - 1)
        in[j] = j > kConvRegs - 1 - p.taps ? *reinterpret_cast<const f32x4*>(p.proj + (size_t)(row0 + j - (kConvRegs - 1)) * p.ld_proj + col) : zero;
#pragma unroll
      for (int g = 0; g < kConvRegs; ++g)      // [tokens back]
        w[g] = g < p.taps ? *reinterpret_cast<const f32x4*>(p.conv_w + (size_t)(p.taps - 1 - g) * p.conv_ch + col) : zero;
#pragma unroll
      for (int r = 0; r < ROWS; ++r)
#pragma unroll
        for (int g = kConvRegs - 1; g >= 0; --g) y[i][r] += w[g] * in[r + kConvRegs - 1 - g];
    }
  } else {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int u = i * NT + tid;
      if (u >= total) continue;
      int block, c;
      const int col = place(u, block, c);
#pragma unroll
      for (int r = 0; r < ROWS; ++r) {
        if (R[r].pos < 0) continue;
        const f32x4 now = input(r, row0 + r, 0, col);
        if (!p.taps) {
          y[i][r] = now;
          continue;
        }
        const float* cw = p.conv_w + (size_t)(p.taps - 1) * p.conv_ch + col;      // (the newest token's)
        for (int g0 = p.taps - 1; g0 >= 0; g0 -= kConvRegs) {      // the oldest first, kConvRegs requested at once
          f32x4 w[kConvRegs], in[kConvRegs];
#pragma unroll
          for (int j = 0; j < kConvRegs; ++j) {
            const int g = g0 - j;
            in[j] = g > 0 ? input(r, row0 + r, g, col) : now;
            w[j] = g >= 0 ? *reinterpret_cast<const f32x4*>(cw - (size_t)(g >= 0 ? g : 0) * p.conv_ch) : zero;
          }
#pragma unroll
          for (int j = 0; j < kConvRegs; ++j) y[i][r] += w[j] * in[j];
        }
        if (p.n_spans == 0)      // segments of one token: nobody else reads this entry of the ring
          *reinterpret_cast<f32x4*>(p.ring + ((size_t)R[r].slot * p.taps + R[r].pos % p.taps) * p.conv_ch + col) = now;
      }
    }
  }
  float inv[2][ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) inv[0][r] = inv[1][r] = 1.f;
  if (p.norm_whole) {
    const int wave = tid >> 6, lane = tid & 63;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      float ss[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int u = i * NT + tid;
        const float s = quad_squares(y[i][r]);
        if (u < quads[0]) ss[0] += s;
        else if (u < quads[0] + quads[1]) ss[1] += s;
      }
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const float s = wave_sum(ss[b]);
        if (lane == 0) red[wave][2 * r + b] = s;
      }
    }
    __syncthreads();
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        float s = 0.f;
#pragma unroll
        for (int w = 0; w < NT / 64; ++w) s += red[w][2 * r + b];
        inv[b][r] = 1.0f / sqrtf(s / (float)n[b] + p.eps);
      }
  }
  const bool whole = p.dim % 4 == 0 && p.vdim % 4 == 0;      // a quad stays in one head
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int u = i * NT + tid;
    if (u >= total) continue;
    int block, c;
    place(u, block, c);
    const float* nw = block == 0 ? p.q_norm : (block == 1 ? p.k_norm : nullptr);
    f32x4 w = {1.f, 1.f, 1.f, 1.f};
    if (nw) w = *reinterpret_cast<const f32x4*>(nw + c);
    const int d = block == 2 ? p.vdim : p.dim, dp = block == 2 ? p.vdim_p : p.dim_p, e0 = c / d, c0 = c - e0 * d;
    CT* pages = reinterpret_cast<CT*>(block == 2 ? p.vcache : p.kcache);
    f32x4 first[ROWS];
    const bool mix = block == 2 && p.vfirst;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) first[r] = mix && !p.vfirst_write && R[r].pos >= 0 ? *reinterpret_cast<const f32x4*>(p.vfirst + (size_t)(row0 + r) * p.ld_vfirst + c) : zero;
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      if (R[r].pos < 0) continue;
      const int row = row0 + r;
      f32x4 v = block == 2 ? y[i][r] : y[i][r] * inv[block & 1][r] * w;
      if (mix) {
        if (p.vfirst_write) *reinterpret_cast<f32x4*>(p.vfirst + (size_t)row * p.ld_vfirst + c) = v;
        else v = (1.f - p.vmix) * v + p.vmix * first[r];
      }
      if (whole) {
        if (block == 0) {
          const float out[4] = {v[0], v[1], v[2], v[3]};
          store_operand4(p.q, row, e0 * p.dim_p + c0, out);
        } else {
          store_page4(pages + (page[r] + ((size_t)e0 << p.log_block)) * dp + c0, v);
        }
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          if (c + k >= n[block]) break;
          const int e = (c + k) / d, cc = c + k - e * d;
          if (block == 0) store_operand(p.q, row, e * p.dim_p + cc, v[k]);
          else pages[(page[r] + ((size_t)e << p.log_block)) * dp + cc] = to_page<CT>(v[k]);
        }
      }
    }
  }
  // padding between heads: queries multiply it, so it must not hold another layer's numbers
  const int pad = p.dim_p - p.dim, vpad = p.vdim_p - p.vdim;
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    if (R[r].pos < 0) continue;
    for (int x = tid; x < (H + G) * pad; x += NT) {
      const int e = x / pad, c = p.dim + x - e * pad;
      if (e < H) store_operand(p.q, row0 + r, e * p.dim_p + c, 0.f);
      else reinterpret_cast<CT*>(p.kcache)[(page[r] + ((size_t)(e - H) << p.log_block)) * p.dim_p + c] = 0;
    }
    for (int x = tid; x < G * vpad; x += NT) {
      const int e = x / vpad;
      reinterpret_cast<CT*>(p.vcache)[(page[r] + ((size_t)e << p.log_block)) * p.vdim_p + p.vdim + x - e * vpad] = 0;
    }
  }
}

// grid (taps - 1, spans, columns / 1024): the inputs that the next step's convolutions read
__global__ __launch_bounds__(256) void window_ring_kernel(ChattsWindowArgs p) {
  const ChattsSpan sp = p.spans[blockIdx.y];
  const int i = blockIdx.x, c = (blockIdx.z * 256 + threadIdx.x) * 4;
  if (i >= sp.t || c >= p.conv_ch) return;
  const int last = sp.t - 1 - i;
  *reinterpret_cast<f32x4*>(p.ring + ((size_t)sp.slot * p.taps + (sp.pos0 + last) % p.taps) * p.conv_ch + c) =
      *reinterpret_cast<const f32x4*>(p.proj + (size_t)(sp.row0 + last) * p.ld_proj + c);
}

// ---- vector units: grid (heads, rows) ----
template <typename CT>
__global__ __launch_bounds__(256) void window_attend_kernel(ChattsWindowArgs p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, hk = h / (p.heads / p.kv_heads);
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  float* sq = sm;              // [dim_p]
  float* sc = sq + p.dim_p;    // [64] scores, then weights
  for (int i = tid; i < p.dim_p; i += 256) {
    const size_t at = (size_t)row * p.q.ld + h * p.dim_p + i;
    sq[i] = p.q.f32 ? p.q.f32[at] : bf16_to_f32(p.q.hi[at]) + (p.q.lo ? bf16_to_f32(p.q.lo[at]) : 0.f);
  }
  float m = p.sink ? 0.f : -INFINITY, l = p.sink ? 1.f : 0.f, o = 0.f;      // column tid
  const WindowTiles T(p, R.pos, R.pos, 6);
  const int n = T.count(), low = window_low(p, R.pos);
  const float slope = p.slopes ? p.slopes[h] : 0.f, r1 = p.log_r1 ? p.log_r1[h] : 0.f, r2 = p.log_r1 ? p.log_r2[h] : 0.f;
  for (int i = 0; i < n; ++i) {
    __syncthreads();
    const int k0 = T.tile(i) * 64;
    const size_t at = window_tile(p, R.slot, hk, k0);
    const CT* kt = reinterpret_cast<const CT*>(p.kcache) + at * p.dim_p;
    const CT* vt = reinterpret_cast<const CT*>(p.vcache) + at * p.vdim_p;
    const int key = tid >> 2, part = tid & 3;
    const bool sees = window_sees(p, R.pos, low, k0 + key);
    float d = 0.f;
    if (sees)
      for (int c = part; c < p.dim_p; c += 4) {
        float kv;
        if constexpr (sizeof(CT) == 4) kv = kt[(size_t)key * p.dim_p + c];
        else kv = bf16_to_f32(kt[(size_t)key * p.dim_p + c]);
        d += kv * sq[c];
      }
    d += lane_xor1(d);
    d += lane_xor2(d);
    d *= p.scale;
    if (p.softcap > 0.f) d = p.softcap * tanhf(d / p.softcap);
    const float far = (float)(R.pos - k0 - key);
    if (part == 0) sc[key] = sees ? d - slope * far - (p.log_r1 ? r1 * log1pf(r2 * far) : 0.f) : -INFINITY;
    __syncthreads();
    const float s = sc[tid & 63];
    const float mn = fmaxf(m, wave_max(s)), safe = mn == -INFINITY ? 0.f : mn;
    const float e = expf(s - safe), alpha = expf(m - safe);
    l = l * alpha + wave_sum(e);
    m = mn;
    __syncthreads();
    if (tid < 64) sc[tid] = e;
    __syncthreads();
    if (tid < p.vdim) {
      const int lim = R.pos + 1 - k0 < 64 ? R.pos + 1 - k0 : 64;
      o *= alpha;
      for (int k = 0; k < lim; ++k) {
        const float w = sc[k];
        if (w == 0.f) continue;      // (uniform)
        if constexpr (sizeof(CT) == 4) o += w * vt[(size_t)k * p.vdim_p + tid];
        else o += w * bf16_to_f32(vt[(size_t)k * p.vdim_p + tid]);
      }
    }
  }
  if (tid < p.vdim) store_operand(p.out, row, h * p.vdim + tid, o / l * window_gate(p, row, h, tid) * p.out_scale);
}

// ---- one row on the matrix pipe: grid (splits, kv heads * head tiles, rows), 4 waves ----
// A wave walks tiles of 32 keys on its own (tiles 4 split + wave, ...): S^T = K Q^T with the key rows straight from memory as A fragments, so that a
// lane ends up with 8 scores of one head (column = lane & 15); O^T = V^T P^T with V through a private piece of LDS (LDS-DMA) and transposing reads - its B
// fragment IS the 8 probabilities of the lane (K slot 8 g + j = key 4 g + j, j < 4, or 16 + 4 g + j - 4, on both sides).  The waves' softmaxes meet once.
template <int NK, int NV, int SCORE>      // dim_p <= 32 NK, vdim_p <= 16 NV
__global__ __launch_bounds__(256, NV <= 4 ? 4 : (NV <= 8 ? 3 : 1)) void window_decode_kernel(ChattsWindowArgs p) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int split = blockIdx.x, row = blockIdx.z, tid = threadIdx.x, lane = tid & 63, fr = lane & 15, fg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const ChattsRow R = p.rows[row];
  if (R.pos < 0) return;
  const int group = p.heads / p.kv_heads, htiles = (group + 15) / 16, hk = blockIdx.y / htiles, h0 = (blockIdx.y - hk * htiles) * 16;
  const int nk = p.dim_p >> 5, nv = p.vdim_p >> 4, ldv = p.vdim_p;
  const int hl = h0 + fr < group ? h0 + fr : group - 1, head = hk * group + hl;
  uint16_t* vs = reinterpret_cast<uint16_t*>(smem) + wave * 32 * ldv;
  bf16x8_t q[NK];
#pragma unroll
  for (int k = 0; k < NK; ++k)
    if (k < nk) q[k] = *reinterpret_cast<const bf16x8_t*>(p.q.hi + (size_t)row * p.q.ld + head * p.dim_p + k * 32 + fg * 8);
  const WindowTiles T(p, R.pos, R.pos, 5);
  const int n = T.count(), stride = 4 * p.n_splits, low = window_low_of<SCORE>(p, R.pos);
  const float slope2 = window_sloped<SCORE>(p) ? p.slopes[head] * kLog2e : 0.f;
  const float r1 = window_logged<SCORE>(p) ? p.log_r1[head] : 0.f, r2 = window_logged<SCORE>(p) ? p.log_r2[head] : 0.f;
  float m = -INFINITY, l = 0.f;
  f32x4 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) o[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const float scale2 = p.scale * kLog2e, cap2 = p.softcap * kLog2e, capk = window_capped<SCORE>(p) ? 2.f * kLog2e * p.scale / p.softcap : 0.f;
  constexpr int VP = NV;      // LDS-DMA requests of a value tile: 64 pieces of 16 bytes each
  // 16-byte piece c of row r lies at position c ^ (r & sw): the transposing reads of neighbouring rows meet different banks
  const int vc = p.vdim_p >> 3, sw = (vc & 7) == 0 ? 7 : ((vc & 3) == 0 ? 3 : 1);
  struct Tile { bf16x8_t k[2][NK]; };
  auto request = [&](int i, Tile& t) __attribute__((always_inline)) {
    const int k0 = T.tile(i) * 32;
    const size_t at = window_tile(p, R.slot, hk, k0);
    const uint16_t* kt = reinterpret_cast<const uint16_t*>(p.kcache) + at * p.dim_p;
    const uint16_t* vt = reinterpret_cast<const uint16_t*>(p.vcache) + at * p.vdim_p;
#pragma unroll
    for (int k = 0; k < NK; ++k)
      if (k < nk) {
        t.k[0][k] = *reinterpret_cast<const bf16x8_t*>(kt + (uint32_t)(fr * p.dim_p + k * 32 + fg * 8));
        t.k[1][k] = *reinterpret_cast<const bf16x8_t*>(kt + (uint32_t)((16 + fr) * p.dim_p + k * 32 + fg * 8));
      }
#pragma unroll
    for (int e = 0; e < VP; ++e)
      if (e * 64 < 32 * vc) {      // (uniform: a tile is a whole number of requests)
        const int x = e * 64 + lane, r = x / vc, c = x - r * vc;
        __builtin_amdgcn_global_load_lds((gptr_t)(vt + (uint32_t)(r * p.vdim_p + ((c ^ (r & sw)) << 3))), (lptr_t)(vs + e * 512), 16, 0, 0);
      }
  };
  auto use = [&](int i, const Tile& t) __attribute__((always_inline)) {
    const int k0 = T.tile(i) * 32;
    f32x4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int k = 0; k < NK; ++k)
      if (k < nk) {
        s[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(t.k[0][k], q[k], s[0], 0, 0, 0);
        s[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(t.k[1][k], q[k], s[1], 0, 0, 0);
      }
    float v[8], mx = -INFINITY;
    if (window_capped<SCORE>(p)) {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = window_cap(s[j >> 2][j & 3], capk, cap2);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = s[j >> 2][j & 3] * scale2;
    }
    const float d0 = (float)(k0 + fg * 4 - R.pos);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int key = k0 + (j >> 2) * 16 + fg * 4 + (j & 3);
      if (SCORE == kSlope || SCORE == kAny) v[j] += slope2 * (d0 + (float)((j >> 2) * 16 + (j & 3)));
      if (window_logged<SCORE>(p)) v[j] -= window_log(r1, r2, -d0 - (float)((j >> 2) * 16 + (j & 3)));      // (NaN only for keys ahead, which are masked)
      if (!window_sees(p, R.pos, low, key)) v[j] = -INFINITY;
      mx = fmaxf(mx, v[j]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx), safe = mn == -INFINITY ? 0.f : mn, alpha = __builtin_amdgcn_exp2f(m - safe);
    m = mn;
    bf16x8_t pf;
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float e = __builtin_amdgcn_exp2f(v[j] - safe);
      sum += e;
      pf[j] = (__bf16)e;
    }
    l = l * alpha + sum;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");      // the values have landed
    const int lim = R.pos + 1 - k0;
    if (lim < 32) {      // rows never written may hold anything: zeros
      for (int x = lim * vc + lane; x < 32 * vc; x += 64) *reinterpret_cast<u32x4*>(vs + x * 8) = (u32x4){0u, 0u, 0u, 0u};
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
    const int tr = fg * 4 + (fr >> 2), swz = tr & sw, cb = (fr >> 1) & 1;
    const uint16_t* t0 = vs + tr * ldv + (fr & 1) * 4;
#pragma unroll
    for (int f = 0; f < NV; ++f)
      if (f < nv) {
        union { w16x4 h[2]; bf16x8_t v; } a;
        a.h[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_w16x4)(t0 + (((2 * f + cb) ^ swz) << 3)));
        a.h[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_w16x4)(t0 + 16 * ldv + (((2 * f + cb) ^ swz) << 3)));
#pragma unroll
        for (int r = 0; r < 4; ++r) o[f][r] *= alpha;
        o[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, pf, o[f], 0, 0, 0);
      }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");      // this tile has been read before the next one is written
  };
  Tile t;
  for (int i = split * 4 + wave; i < n; i += stride) {
    request(i, t);
    use(i, t);
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  // the four waves meet: [wave][16 heads][vdim_p + 4]
  __syncthreads();
  float* part = reinterpret_cast<float*>(smem);
  const int ldp = p.vdim_p + 4;
#pragma unroll
  for (int f = 0; f < NV; ++f)
    if (f < nv) *reinterpret_cast<f32x4*>(part + (wave * 16 + fr) * ldp + f * 16 + fg * 4) = o[f];
  if (fg == 0) {
    part[(wave * 16 + fr) * ldp + p.vdim_p] = m;
    part[(wave * 16 + fr) * ldp + p.vdim_p + 1] = l;
  }
  __syncthreads();
  const bool whole = p.n_splits == 1;
  const int hn = group - h0 < 16 ? group - h0 : 16;
  for (int x = tid; x < hn * p.vdim_p; x += 256) {
    const int hh = x / p.vdim_p, c = x - hh * p.vdim_p;
    const int hd = hk * group + h0 + hh;
    float mw[4], M = whole && p.sink ? 0.f : -INFINITY;
#pragma unroll
    for (int w = 0; w < 4; ++w) { mw[w] = part[(w * 16 + hh) * ldp + p.vdim_p]; M = fmaxf(M, mw[w]); }
    const float safe = M == -INFINITY ? 0.f : M;
    float L = whole && p.sink ? __builtin_amdgcn_exp2f(-safe) : 0.f, acc = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f(mw[w] - safe);
      L += f * part[(w * 16 + hh) * ldp + p.vdim_p + 1];
      acc += f * part[(w * 16 + hh) * ldp + c];
    }
    if (whole) {
      if (c < p.vdim) store_operand(p.out, row, hd * p.vdim + c, acc / L * window_gate(p, row, hd, c) * p.out_scale);
    } else {
      float* dst = p.partial + (((size_t)row * p.heads + hd) * p.n_splits + split) * ldp;
      dst[c] = acc;
      if (c == 0) { dst[p.vdim_p] = M; dst[p.vdim_p + 1] = L; }
    }
  }
}

// merge of the splits: grid (heads, rows)
__global__ __launch_bounds__(128) void window_merge_kernel(ChattsWindowArgs p) {
  __shared__ float w[64];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, ld = p.vdim_p + 4;
  if (p.rows[row].pos < 0) return;
  const float* part = p.partial + ((size_t)row * p.heads + h) * p.n_splits * ld;
  if (tid < 64) {
    const float m = tid < p.n_splits ? part[(size_t)tid * ld + p.vdim_p] : -INFINITY, l = tid < p.n_splits ? part[(size_t)tid * ld + p.vdim_p + 1] : 0.f;
    float M = wave_max(m);
    if (p.sink) M = fmaxf(M, 0.f);
    const float f = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - M);
    const float L = wave_sum(f * l) + (p.sink ? __builtin_amdgcn_exp2f(-M) : 0.f);
    w[tid] = f / L;
  }
  __syncthreads();
  for (int c = tid; c < p.vdim; c += 128) {
    float o = 0.f;
#pragma unroll 4
    for (int s = 0; s < p.n_splits; ++s) o += w[s] * part[(size_t)s * ld + c];
    store_operand(p.out, row, h * p.vdim + c, o * window_gate(p, row, h, c) * p.out_scale);
  }
}

// ---- many rows: grid (heads, query tiles of 128, spans); a wave owns 32 queries of one head, 64 keys per step ----
// S^T = K Q^T, O^T = V^T P^T as above; keys and values of a tile are staged by all waves, the next tile's requested while this one is multiplied.
template <int NK, int NV, int OCC, int SCORE>      // dim_p <= 32 NK, vdim_p <= 16 NV
__global__ __launch_bounds__(256, OCC) void window_prefill_kernel(ChattsWindowArgs p) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const ChattsSpan sp = p.spans[blockIdx.z];
  const int qt0 = (gridDim.y - 1 - blockIdx.y) * 128, h = blockIdx.x, hk = h / (p.heads / p.kv_heads);
  if (qt0 >= sp.t) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fr = lane & 15, fg = lane >> 4;
  const int dq = p.dim_p, ldk = dq + 8, ldv = p.vdim_p + 16, nk = dq >> 5, nv = p.vdim_p >> 4;
  uint16_t* ks = reinterpret_cast<uint16_t*>(smem);      // [64][ldk]
  uint16_t* vs = ks + 64 * ldk;                          // [64][ldv]
  const int qlast = qt0 + 127 < sp.t ? qt0 + 127 : sp.t - 1;
  const WindowTiles T(p, sp.pos0 + qt0, sp.pos0 + qlast, 6);
  const int n = T.count(), plast = sp.pos0 + qlast;
  const int q0 = qt0 + wave * 32, w0 = sp.pos0 + q0, w1 = w0 + 31 < plast ? w0 + 31 : plast;      // this wave's positions
  bf16x8_t q[2][NK];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    int r = q0 + u * 16 + fr;
    if (r > sp.t - 1) r = sp.t - 1;
    const uint16_t* src = p.q.hi + (size_t)(sp.row0 + r) * p.q.ld + h * dq + fg * 8;
#pragma unroll
    for (int k = 0; k < NK; ++k)
      if (k < nk) q[u][k] = *reinterpret_cast<const bf16x8_t*>(src + k * 32);
  }
  f32x4 o[NV][2];
#pragma unroll
  for (int i = 0; i < NV; ++i) o[i][0] = o[i][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const float m0 = p.sink ? 0.f : -INFINITY, l0 = p.sink && fg == 0 ? 1.f : 0.f;
  float m[2] = {m0, m0}, l[2] = {l0, l0};
  const float scale2 = p.scale * kLog2e;      // scores in base 2
  const float cap2 = p.softcap * kLog2e, capk = window_capped<SCORE>(p) ? 2.f * kLog2e * p.scale / p.softcap : 0.f;
  const float slope2 = window_sloped<SCORE>(p) ? p.slopes[h] * kLog2e : 0.f;
  const float r1 = window_logged<SCORE>(p) ? p.log_r1[h] : 0.f, r2 = window_logged<SCORE>(p) ? p.log_r2[h] : 0.f;
  const int low_first = window_low_of<SCORE>(p, w0), low_last = window_low_of<SCORE>(p, w1);
  int lows[2] = {0, 0};
  if (SCORE == kCap || SCORE == kAny) { lows[0] = window_low(p, w0 + fr); lows[1] = window_low(p, w0 + 16 + fr); }
  const bool masked = window_masked(p);
  constexpr int KP = NK, VP = (NV + 1) / 2;
  u32x4 rk[KP], rv[VP];
  const int kc = dq >> 3, vc = p.vdim_p >> 3;
  auto fetch = [&](int i) __attribute__((always_inline)) {
    const int k0 = T.tile(i) * 64;
    const size_t at = window_tile(p, sp.slot, hk, k0);
    const uint16_t* kt = reinterpret_cast<const uint16_t*>(p.kcache) + at * dq;
    const uint16_t* vt = reinterpret_cast<const uint16_t*>(p.vcache) + at * p.vdim_p;
#pragma unroll
    for (int e = 0; e < KP; ++e) {
      const int x = e * 256 + tid;
      if (x < 64 * kc) rk[e] = *reinterpret_cast<const u32x4*>(kt + (size_t)x * 8);
    }
#pragma unroll
    for (int e = 0; e < VP; ++e) {
      const int x = e * 256 + tid;
      rv[e] = (u32x4){0u, 0u, 0u, 0u};
      if (x < 64 * vc && k0 + x / vc <= plast) rv[e] = *reinterpret_cast<const u32x4*>(vt + (size_t)x * 8);      // (a row never written may hold anything)
    }
  };
  fetch(0);
  for (int i = 0; i < n; ++i) {
    __syncthreads();
#pragma unroll
    for (int e = 0; e < KP; ++e) {
      const int x = e * 256 + tid, r = x / kc;
      if (x < 64 * kc) *reinterpret_cast<u32x4*>(ks + r * ldk + (x - r * kc) * 8) = rk[e];
    }
#pragma unroll
    for (int e = 0; e < VP; ++e) {
      const int x = e * 256 + tid, r = x / vc;
      if (x < 64 * vc) *reinterpret_cast<u32x4*>(vs + r * ldv + (x - r * vc) * 8) = rv[e];
    }
    __syncthreads();
    if (i + 1 < n) fetch(i + 1);
    const int k0 = T.tile(i) * 64;
    // (uniform per wave) nothing of the tile is visible to this wave's queries
    if (k0 > w1 || w0 > w1 || (masked && k0 + 63 < low_first && k0 >= p.keep_first)) continue;
    const bool edge = k0 + 63 > w0 || (masked && k0 < low_last && k0 + 63 >= p.keep_first);      // some key is hidden from some query
    f32x4 s[4][2];      // [16-key block][query block]
#pragma unroll
    for (int a = 0; a < 4; ++a) s[a][0] = s[a][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const uint16_t* kb = ks + fr * ldk + fg * 8;
    {
      bf16x8_t kf[2][4];
      auto request = [&](int k, bf16x8_t (&dst)[4]) __attribute__((always_inline)) {
#pragma unroll
        for (int a = 0; a < 4; ++a) dst[a] = *reinterpret_cast<const bf16x8_t*>(kb + a * 16 * ldk + k * 32);
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
      const int qpos = w0 + u * 16 + fr, low = SCORE == kCap || SCORE == kAny ? lows[u] : window_low_of<SCORE>(p, qpos);
      if (window_capped<SCORE>(p)) {
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
          for (int r = 0; r < 4; ++r) s[a][u][r] = window_cap(s[a][u][r], capk, cap2);
      } else {
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
          for (int r = 0; r < 4; ++r) s[a][u][r] *= scale2;
      }
      if (window_sloped<SCORE>(p)) {
        const float d0 = (float)(k0 + fg * 4 - qpos);
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
          for (int r = 0; r < 4; ++r) s[a][u][r] += slope2 * (d0 + (float)(a * 16 + r));
      }
      if (window_logged<SCORE>(p)) {
        const float d0 = (float)(qpos - k0 - fg * 4);
#pragma unroll
        for (int a = 0; a < 4; ++a)
#pragma unroll
          for (int r = 0; r < 4; ++r) s[a][u][r] -= window_log(r1, r2, d0 - (float)(a * 16 + r));      // (NaN only for keys ahead, which are masked)
      }
      float mx = -INFINITY;
#pragma unroll
      for (int a = 0; a < 4; ++a)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float v = s[a][u][r];
          if (edge && !window_sees(p, qpos, low, k0 + a * 16 + fg * 4 + r)) v = -INFINITY;
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
        for (int f = 0; f < NV; ++f)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[f][u][r] *= alpha;
      }
    }
    {
      // transposing reads: lane -> rows 4 g + (fr >> 2) (and + 16) of a 32-key group, 4 columns of the fragment's 16
      const uint16_t* t0 = vs + (fg * 4 + (fr >> 2)) * ldv + (fr & 3) * 4;
      union Tr { w16x4 h[2]; bf16x8_t v; };
      Tr vf[2][2];
      auto request = [&](int f, Tr (&dst)[2]) __attribute__((always_inline)) {
#pragma unroll
        for (int g = 0; g < 2; ++g) {
          dst[g].h[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_w16x4)(t0 + g * 32 * ldv + f * 16));
          dst[g].h[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_w16x4)(t0 + (g * 32 + 16) * ldv + f * 16));
        }
      };
      request(0, vf[0]);
#pragma unroll
      for (int f = 0; f < NV; ++f)
        if (f < nv) {
          if (f + 1 < NV && f + 1 < nv) request(f + 1, vf[(f + 1) & 1]);
          __builtin_amdgcn_sched_barrier(0);
#pragma unroll
          for (int g = 0; g < 2; ++g) {
            o[f][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[f & 1][g].v, pf[g][0], o[f][0], 0, 0, 0);
            o[f][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[f & 1][g].v, pf[g][1], o[f][1], 0, 0, 0);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
    }
  }
  const bool quads = p.vdim % 4 == 0 && (p.off_gate < 0 || p.gate_heads || p.off_gate % 4 == 0) && p.out.ld % 4 == 0;
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int r = q0 + u * 16 + fr;
    float L = l[u];
    L += __shfl_xor(L, 16, 64);
    L += __shfl_xor(L, 32, 64);
    if (r >= sp.t) continue;
    const size_t row = sp.row0 + r;
    const float inv = 1.0f / L * p.out_scale * (p.gate_heads ? window_gate(p, row, h, 0) : 1.f);
#pragma unroll
    for (int f = 0; f < NV; ++f) {
      const int c = f * 16 + fg * 4, at = h * p.vdim + c;
      if (f >= nv || c >= p.vdim) continue;
      if (quads) {
        f32x4 g = {1.f, 1.f, 1.f, 1.f};
        if (p.off_gate >= 0 && !p.gate_heads) {
          g = *reinterpret_cast<const f32x4*>(p.proj + row * p.ld_proj + p.off_gate + at);
#pragma unroll
          for (int k = 0; k < 4; ++k) g[k] = sigmoid_f(g[k]);
        }
        const float v[4] = {o[f][u][0] * inv * g[0], o[f][u][1] * inv * g[1], o[f][u][2] * inv * g[2], o[f][u][3] * inv * g[3]};
        store_operand4(p.out, row, at, v);
      } else {
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (c + k < p.vdim) store_operand(p.out, row, at + k, o[f][u][k] * inv * (p.gate_heads ? 1.f : window_gate(p, row, h, c + k)));
      }
    }
  }
}

static int check_window(const ChattsWindowArgs* a, const char* who) {
  CHATTS_REQUIRE(a && a->proj && a->kcache && a->vcache && a->table && a->rows && (a->q_norm != nullptr) == (a->k_norm != nullptr) && (a->q.f32 || a->q.hi), CHATTS_E_BADARG, "%s: null pointer", who);
  CHATTS_REQUIRE(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->dim >= 1 && a->dim <= a->dim_p && a->dim_p <= 256 && a->dim_p % 32 == 0 &&
                     a->vdim >= 1 && a->vdim <= a->vdim_p && a->vdim_p <= 256 && a->vdim_p % 16 == 0, CHATTS_E_SHAPE, "%s: heads %d / %d of %d, %d (at most 256)", who,
                 a->heads, a->kv_heads, a->dim, a->vdim);
  CHATTS_REQUIRE(a->off_q >= 0 && a->off_k >= 0 && a->off_v >= 0 && a->off_q + a->heads * a->dim <= a->ld_proj && a->off_k + a->kv_heads * a->dim <= a->ld_proj &&
                     a->off_v + a->kv_heads * a->vdim <= a->ld_proj && a->off_gate + (a->gate_heads ? a->heads : a->heads * a->vdim) <= a->ld_proj &&
                     a->ld_proj % 4 == 0, CHATTS_E_SHAPE, "%s: column blocks", who);
  CHATTS_REQUIRE(a->n_rows >= 0 && a->n_rows <= 65535, CHATTS_E_SHAPE, "%s: %d rows", who, a->n_rows);
  CHATTS_REQUIRE(a->log_block >= 6 && a->log_block <= 15 && a->window >= 0 && a->keep_first >= 0, CHATTS_E_SHAPE, "%s: pages of 2^%d tokens, window %d, kept %d", who,
                 a->log_block, a->window, a->keep_first);
  CHATTS_REQUIRE(a->chunk >= 0 && (a->chunk == 0 || a->window == 0) && a->softcap >= 0.f && (!a->gate_heads || a->off_gate >= 0), CHATTS_E_SHAPE,
                 "%s: window %d and chunks of %d, scores capped at %g", who, a->window, a->chunk, (double)a->softcap);
  CHATTS_REQUIRE((a->log_r1 != nullptr) == (a->log_r2 != nullptr), CHATTS_E_BADARG, "%s: half of a logarithmic bias", who);
  CHATTS_REQUIRE(a->rot >= 0 && a->rot % 2 == 0 && a->rot <= a->dim && (a->rot == 0 || (a->cos_tab && a->sin_tab)), CHATTS_E_SHAPE, "%s: %d of %d dimensions rotated", who,
                 a->rot, a->dim);
  CHATTS_REQUIRE(a->taps >= 0 && (a->taps == 0 || (a->conv_w && a->ring && a->conv_ch % 4 == 0 && a->conv_ch <= a->ld_proj && a->off_q + a->heads * a->dim <= a->conv_ch &&
                                                   a->off_k + a->kv_heads * a->dim <= a->conv_ch && a->off_v + a->kv_heads * a->vdim <= a->conv_ch)),
                 CHATTS_E_SHAPE, "%s: convolutions over %d tokens of %d columns", who, a->taps, a->conv_ch);
  CHATTS_REQUIRE(!a->vfirst || (a->ld_vfirst >= a->kv_heads * a->vdim && a->ld_vfirst % 4 == 0 && ((uintptr_t)a->vfirst % 16) == 0), CHATTS_E_SHAPE,
                 "%s: rows of %d first values", who, a->ld_vfirst);
  const bool rows = a->taps > 0 || a->norm_whole;
  CHATTS_REQUIRE(!rows || (!a->rot && !a->unit && (!a->q_norm || a->norm_whole)), CHATTS_E_SHAPE, "%s: convolutions and norms over all heads do not combine with per-head steps", who);
  CHATTS_REQUIRE(!rows || (a->off_q % 4 == 0 && a->off_k % 4 == 0 && a->off_v % 4 == 0 && (!a->norm_whole || (a->q_norm && ((uintptr_t)a->q_norm % 16) == 0 &&
                           ((uintptr_t)a->k_norm % 16) == 0)) && (((uintptr_t)a->conv_w | (uintptr_t)a->ring) % 16) == 0 &&
                           a->heads * a->dim + a->kv_heads * (a->dim + a->vdim) + 12 <= 32768 && a->off_q + (a->heads * a->dim + 3) / 4 * 4 <= a->ld_proj &&
                           a->off_k + (a->kv_heads * a->dim + 3) / 4 * 4 <= a->ld_proj && a->off_v + (a->kv_heads * a->vdim + 3) / 4 * 4 <= a->ld_proj), CHATTS_E_SHAPE,
                 "%s: %d + %d heads by whole rows", who, a->heads, a->kv_heads);
  CHATTS_REQUIRE((((uintptr_t)a->kcache | (uintptr_t)a->vcache | (uintptr_t)a->proj) % 16) == 0 && a->q.ld >= a->heads * a->dim_p && a->q.ld % 8 == 0 &&
                     (a->cache_f32 ? a->q.f32 != nullptr : a->q.hi != nullptr), CHATTS_E_SHAPE, "%s: alignment / queries", who);
  return CHATTS_OK;
}
static ChattsWindowArgs window_scaled(const ChattsWindowArgs* args) {      // out_scale 0: 1
  ChattsWindowArgs a = *args;
  if (a.out_scale == 0.f) a.out_scale = 1.f;
  return a;
}
static bool window_out_ok(const ChattsWindowArgs* a) { return (a->out.f32 || a->out.hi) && a->out.ld >= a->heads * a->vdim; }

template <typename CT>
static void launch_window_quads(const ChattsWindowArgs* a, int heads, int widest, hipStream_t s) {
  const int lph = widest <= 64 ? 16 : (widest <= 128 ? 32 : 64), groups = (heads * lph + 255) / 256;      // workgroups that would take one group of heads per wave
  const dim3 g(a->n_rows, a->n_rows <= 64 ? groups : (groups + 1) / 2), b(256);
  if (lph == 16) hipLaunchKernelGGL((window_prep_quads_kernel<CT, 16>), g, b, 0, s, *a);
  else if (lph == 32) hipLaunchKernelGGL((window_prep_quads_kernel<CT, 32>), g, b, 0, s, *a);
  else hipLaunchKernelGGL((window_prep_quads_kernel<CT, 64>), g, b, 0, s, *a);
}

template <typename CT>
static int launch_window_rows(const ChattsWindowArgs* a, hipStream_t s) {
  const int quads = (a->heads * a->dim + 3) / 4 + (a->kv_heads * a->dim + 3) / 4 + (a->kv_heads * a->vdim + 3) / 4;
  if (a->n_rows > 64 && quads <= 4 * 512) hipLaunchKernelGGL((window_prep_rows_kernel<CT, 512, 4, 4>), dim3((a->n_rows + 3) / 4), dim3(512), 0, s, *a);
  else if (quads <= 2 * 1024) hipLaunchKernelGGL((window_prep_rows_kernel<CT, 1024, 2, 1>), dim3(a->n_rows), dim3(1024), 0, s, *a);
  else hipLaunchKernelGGL((window_prep_rows_kernel<CT, 1024, 8, 1>), dim3(a->n_rows), dim3(1024), 0, s, *a);
  if (a->n_spans > 0 && a->taps > 1)
    hipLaunchKernelGGL(window_ring_kernel, dim3(a->taps - 1, a->n_spans, (a->conv_ch + 1023) / 1024), dim3(256), 0, s, *a);
  CHATTS_CHECK_LAUNCH("window_prep_rows");
  return CHATTS_OK;
}

template <typename K>
static int window_lds(K kernel, size_t bytes, bool& done) {
  if (!done) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    CHATTS_REQUIRE(e == hipSuccess, CHATTS_E_LAUNCH, "window attention: cannot reserve LDS: %s", hipGetErrorString(e));
    done = true;
  }
  return CHATTS_OK;
}

static int window_score(const ChattsWindowArgs* a) {
  if (a->softcap > 0.f && !a->slopes && !a->log_r1) return kCap;
  if (a->softcap > 0.f || a->chunk > 0 || (a->slopes && a->log_r1)) return kAny;
  return a->log_r1 ? kLog : (a->slopes ? kSlope : kPlain);
}

template <int NK, int NV, int SCORE>
static int launch_window_decode_as(const ChattsWindowArgs* a, hipStream_t s) {
  static bool done = false;
  const size_t most = (size_t)4 * 16 * (NV * 16 + 4) * 4;      // the waves' meeting; their value tiles (4 x 32 x vdim_p bf16) are smaller
  if (const int rc = window_lds(&window_decode_kernel<NK, NV, SCORE>, most, done)) return rc;
  const int group = a->heads / a->kv_heads;
  hipLaunchKernelGGL((window_decode_kernel<NK, NV, SCORE>), dim3(a->n_splits, a->kv_heads * ((group + 15) / 16), a->n_rows), dim3(256),
                     (size_t)4 * 16 * (a->vdim_p + 4) * 4, s, *a);
  CHATTS_CHECK_LAUNCH("window_decode");
  return CHATTS_OK;
}
template <int NK, int NV>
static int launch_window_decode(const ChattsWindowArgs* a, hipStream_t s) {
  switch (window_score(a)) {
    case kPlain: return launch_window_decode_as<NK, NV, kPlain>(a, s);
    case kSlope: return launch_window_decode_as<NK, NV, kSlope>(a, s);
    case kCap: return launch_window_decode_as<NK, NV, kCap>(a, s);
    case kLog: return launch_window_decode_as<NK, NV, kLog>(a, s);
    default: return launch_window_decode_as<NK, NV, kAny>(a, s);
  }
}
template <int NK, int NV, int OCC, int SCORE>
static int launch_window_prefill_as(const ChattsWindowArgs* a, hipStream_t s) {
  static bool done = false;
  if (const int rc = window_lds(&window_prefill_kernel<NK, NV, OCC, SCORE>, (size_t)64 * (NK * 32 + 8 + NV * 16 + 16) * 2, done)) return rc;
  hipLaunchKernelGGL((window_prefill_kernel<NK, NV, OCC, SCORE>), dim3(a->heads, (a->longest + 127) / 128, a->n_spans), dim3(256),
                     (size_t)64 * (a->dim_p + 8 + a->vdim_p + 16) * 2, s, *a);
  CHATTS_CHECK_LAUNCH("window_prefill");
  return CHATTS_OK;
}
template <int NK, int NV, int OCC>
static int launch_window_prefill(const ChattsWindowArgs* a, hipStream_t s) {
  switch (window_score(a)) {
    case kPlain: return launch_window_prefill_as<NK, NV, OCC, kPlain>(a, s);
    case kSlope: return launch_window_prefill_as<NK, NV, OCC, kSlope>(a, s);
    case kCap: return launch_window_prefill_as<NK, NV, OCC, kCap>(a, s);
    case kLog: return launch_window_prefill_as<NK, NV, OCC, kLog>(a, s);
    default: return launch_window_prefill_as<NK, NV, OCC, kAny>(a, s);
  }
}

}  // namespace chatts

using namespace chatts;

extern "C" int chatts_window_prep(const ChattsWindowArgs* a, chatts_stream_t stream) {
  if (const int rc = check_window(a, "window_prep")) return rc;
  if (a->n_rows == 0) return CHATTS_OK;
  if (a->taps > 0 || a->norm_whole) return a->cache_f32 ? launch_window_rows<float>(a, as_stream(stream)) : launch_window_rows<uint16_t>(a, as_stream(stream));
  const int heads = a->heads + 2 * a->kv_heads, widest = a->dim > a->vdim ? a->dim : a->vdim;
  if ((a->dim | a->vdim | a->off_q | a->off_k | a->off_v) % 4 == 0 && ((uintptr_t)a->q_norm | (uintptr_t)a->k_norm) % 16 == 0) {
    if (a->cache_f32) launch_window_quads<float>(a, heads, widest, as_stream(stream));
    else launch_window_quads<uint16_t>(a, heads, widest, as_stream(stream));
    CHATTS_CHECK_LAUNCH("window_prep_quads");
    return CHATTS_OK;
  }
  int per_row = (heads + 3) / 4;
  if (per_row > 8192 / a->n_rows) per_row = 8192 / a->n_rows > 1 ? 8192 / a->n_rows : 1;
  if (a->cache_f32) hipLaunchKernelGGL(window_prep_kernel<float>, dim3(a->n_rows, per_row), dim3(256), 0, as_stream(stream), *a);
  else hipLaunchKernelGGL(window_prep_kernel<uint16_t>, dim3(a->n_rows, per_row), dim3(256), 0, as_stream(stream), *a);
  CHATTS_CHECK_LAUNCH("window_prep");
  return CHATTS_OK;
}

extern "C" int chatts_window_can_prefill(int dim_p, int vdim_p) { return dim_p <= 256 && vdim_p <= 256; }

extern "C" int chatts_window_attend(const ChattsWindowArgs* args, chatts_stream_t stream) {
  if (const int rc = check_window(args, "window_attend")) return rc;
  const ChattsWindowArgs scaled = window_scaled(args), *a = &scaled;
  CHATTS_REQUIRE(window_out_ok(a), CHATTS_E_BADARG, "window_attend: no output");
  if (a->n_rows == 0) return CHATTS_OK;
  hipStream_t s = as_stream(stream);
  if (a->cache_f32) {
    hipLaunchKernelGGL(window_attend_kernel<float>, dim3(a->heads, a->n_rows), dim3(256), (size_t)(a->dim_p + 64) * sizeof(float), s, *a);
    CHATTS_CHECK_LAUNCH("window_attend");
    return CHATTS_OK;
  }
  CHATTS_REQUIRE(a->n_splits >= 1 && a->n_splits <= 64 && (a->n_splits == 1 || a->partial), CHATTS_E_BADARG, "window_attend: %d splits", a->n_splits);
  int rc;
  if (a->dim_p <= 64 && a->vdim_p <= 64) rc = launch_window_decode<2, 4>(a, s);
  else if (a->dim_p <= 128 && a->vdim_p <= 128) rc = launch_window_decode<4, 8>(a, s);
  else rc = launch_window_decode<8, 16>(a, s);
  if (rc) return rc;
  if (a->n_splits > 1) {
    hipLaunchKernelGGL(window_merge_kernel, dim3(a->heads, a->n_rows), dim3(128), 0, s, *a);
    CHATTS_CHECK_LAUNCH("window_merge");
  }
  return CHATTS_OK;
}

extern "C" int chatts_window_prefill(const ChattsWindowArgs* args, chatts_stream_t stream) {
  if (const int rc = check_window(args, "window_prefill")) return rc;
  const ChattsWindowArgs scaled = window_scaled(args), *a = &scaled;
  CHATTS_REQUIRE(window_out_ok(a) && a->spans && !a->cache_f32, CHATTS_E_BADARG, "window_prefill: bad arguments");
  if (a->n_rows == 0 || a->n_spans == 0 || a->longest == 0) return CHATTS_OK;
  if (a->dim_p <= 64 && a->vdim_p <= 64) return launch_window_prefill<2, 4, 2>(a, as_stream(stream));
  if (a->dim_p <= 128 && a->vdim_p <= 128) return launch_window_prefill<4, 8, 2>(a, as_stream(stream));
  return launch_window_prefill<8, 16, 1>(a, as_stream(stream));
}
