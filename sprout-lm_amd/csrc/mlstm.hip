// A matrix memory with exponential gates (mLSTM): per head S <- a S + b v k^T, n <- a n + b k, read as S q / max(|n . q|, e^-m).
//
// Gates are kept as logarithms: i = cap tanh(./cap), f = logsigmoid(cap tanh(./cap)), and a running maximum m = max(f + m, i)
// keeps a = exp(f + m_before - m) and b = exp(i - m) at most one.  All of this, the memory and every sum are float32 (running
// sums of logarithms within a chunk float64); only what the projections left is read in the storage type.
//
// The memory of a request and head is [vdim + 1][dim]: a row per value number, the normaliser n as the last row (n is what a
// value number that is always one would leave), so that what walks the memory walks both.
//
// Single tokens and short portions: a block per request and head with the memory in registers (mlstm_step_kernel).  Long
// portions in bfloat16: chunks of 64 tokens side by side, see below.  Everything else: mlstm_general_kernel.
#include "mfma.h"
#include "recurrent.h"
#include "sprout_hip.h"

namespace sprout {

struct MlstmArgs {
  const void* proj;            // [T, stride]: q, k (heads * dim), v, gate (heads * vdim), i, f (heads) at their offsets
  long long stride;
  int q_off, k_off, v_off, gate_off, i_off, f_off;
  int heads, dim, vdim;
  float cap;
  const float *bias_i, *bias_f, *norm;
  float eps;
  const int32_t *q_start, *q_len, *state_slots;
  float* memory;               // [slots, heads, vdim + 1, dim]
  float* maxima;               // [slots, heads]
  void* out;                   // rows of out_stride numbers, the first heads * vdim of a row
  long long out_stride;
};

__device__ __forceinline__ float log_input_gate(float x, float bias, float cap) { return cap * tanhf((x + bias) / cap); }
__device__ __forceinline__ float log_forget_gate(float x, float bias, float cap) {
  const float z = cap * tanhf((x + bias) / cap);
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}
constexpr float kShareFloor = 1e-6f;      // beside max(|n . q|, e^-m)

// Four neighbouring numbers as floats.
__device__ __forceinline__ float4 load_four(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 load_four(const bf16_t* p) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                     __uint_as_float(v.y & 0xffff0000u));
}
__device__ __forceinline__ float dot4(float4 a, float4 b) { return fmaf(a.x, b.x, fmaf(a.y, b.y, fmaf(a.z, b.z, a.w * b.w))); }

// A block per (request, head), token after token.  `lanes` neighbouring lanes (a power of two) hold a row of the memory, four
// numbers each, so that a row's product with q is a sum over those lanes; a block holds threads / lanes rows at a time, NR times.
// Every group of lanes keeps the normaliser for itself.
template <typename T, int NR>
__global__ __launch_bounds__(1024) void mlstm_step_kernel(MlstmArgs a, int lanes) {
  extern __shared__ __attribute__((aligned(16))) float lds[];      // o [2][vdim]
  __shared__ float scratch[16];
  const int s = blockIdx.x, h = blockIdx.y, D = a.dim, V = a.vdim, threads = blockDim.x, R = threads / lanes;
  const int group = threadIdx.x / lanes, l = threadIdx.x % lanes, d0 = 4 * l;
  const bool in = d0 < D;
  const int start = a.q_start[s], n = a.q_len[s], slot = a.state_slots[s];
  float* kept = a.memory + (size_t(slot) * a.heads + h) * size_t(V + 1) * D + (in ? d0 : 0);
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 S[NR], norm = in ? load_four(kept + size_t(V) * D) : zero;
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    const int v = group + r * R;
    S[r] = in && v < V ? load_four(kept + size_t(v) * D) : zero;
  }
  float m = a.maxima[size_t(slot) * a.heads + h];
  const float q_scale = 1.0f / sqrtf(float(D)), bias_i = a.bias_i[h], bias_f = a.bias_f[h];
  T* out = (T*)a.out;
  for (int t = start; t < start + n; ++t) {
    const T* row = (const T*)a.proj + size_t(t) * a.stride;
    // asked for here, before anything waits: what the end of the token needs
    const int v0 = threadIdx.x;
    const float gate0 = v0 < V ? to_float(row[a.gate_off + h * V + v0]) : 0.f, weight0 = v0 < V ? a.norm[h * V + v0] : 0.f;
    const float i = log_input_gate(to_float(row[a.i_off + h]), bias_i, a.cap);
    const float f = log_forget_gate(to_float(row[a.f_off + h]), bias_f, a.cap);
    const float4 q = in ? load_four(row + a.q_off + h * D + d0) : zero, k = in ? load_four(row + a.k_off + h * D + d0) : zero;
    float value[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const int v = group + r * R;
      value[r] = v < V ? to_float(row[a.v_off + h * V + v]) : 0.f;
    }
    const float top = fmaxf(f + m, i), keep = expf(f + m - top), take = expf(i - top);
    m = top;
    norm = make_float4(fmaf(keep, norm.x, take * k.x), fmaf(keep, norm.y, take * k.y), fmaf(keep, norm.z, take * k.z),
                       fmaf(keep, norm.w, take * k.w));
    float nq = dot4(norm, q), o[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const float tv = take * value[r];
      S[r] = make_float4(fmaf(keep, S[r].x, tv * k.x), fmaf(keep, S[r].y, tv * k.y), fmaf(keep, S[r].z, tv * k.z),
                         fmaf(keep, S[r].w, tv * k.w));
      o[r] = dot4(S[r], q);
    }
    for (int off = lanes >> 1; off > 0; off >>= 1) {
      nq += __shfl_xor(nq, off, 64);
#pragma unroll
      for (int r = 0; r < NR; ++r) o[r] += __shfl_xor(o[r], off, 64);
    }
    const float share = q_scale / (fmaxf(fabsf(nq * q_scale), expf(-m)) + kShareFloor);
    float* o_row = lds + ((t - start) & 1) * V;
    float squares = 0.f;
    if (l == 0) {
#pragma unroll
      for (int r = 0; r < NR; ++r) {
        const int v = group + r * R;
        const float x = o[r] * share;
        if (v < V) { o_row[v] = x; squares = fmaf(x, x, squares); }
      }
    }
    squares = block_sum(squares, scratch);      // (its barriers also publish o_row)
    const float unit = 1.0f / sqrtf(squares / float(V) + a.eps);
    T* dst = out + size_t(t) * a.out_stride + h * V;
    if (v0 < V) dst[v0] = from_float<T>(((o_row[v0] * unit) * weight0) * sigmoid(gate0));
    for (int v = v0 + threads; v < V; v += threads)
      dst[v] = from_float<T>(((o_row[v] * unit) * a.norm[h * V + v]) * sigmoid(to_float(row[a.gate_off + h * V + v])));
  }
  if (in) {
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const int v = group + r * R;
      if (v < V) *reinterpret_cast<float4*>(kept + size_t(v) * D) = S[r];
    }
    if (group == 0) *reinterpret_cast<float4*>(kept + size_t(V) * D) = norm;
  }
  if (threadIdx.x == 0) a.maxima[size_t(slot) * a.heads + h] = m;
}

// The same for heads whose memory does not fit a block's registers: it passes through them for every token, NR rows of a group
// at a time, the next rows on their way while these are used.
template <typename T, int NR>
__global__ __launch_bounds__(1024) void mlstm_stream_kernel(MlstmArgs a, int lanes) {
  extern __shared__ __attribute__((aligned(16))) float lds[];      // o [2][vdim]
  __shared__ float scratch[16];
  const int s = blockIdx.x, h = blockIdx.y, D = a.dim, V = a.vdim, threads = blockDim.x, R = threads / lanes;
  const int group = threadIdx.x / lanes, l = threadIdx.x % lanes, d0 = 4 * l;
  const bool in = d0 < D;
  const int start = a.q_start[s], n = a.q_len[s], slot = a.state_slots[s];
  float* kept = a.memory + (size_t(slot) * a.heads + h) * size_t(V + 1) * D + (in ? d0 : 0);
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 norm = in ? load_four(kept + size_t(V) * D) : zero;
  float m = a.maxima[size_t(slot) * a.heads + h];
  const float q_scale = 1.0f / sqrtf(float(D)), bias_i = a.bias_i[h], bias_f = a.bias_f[h];
  T* out = (T*)a.out;
  for (int t = start; t < start + n; ++t) {
    const T* row = (const T*)a.proj + size_t(t) * a.stride;
    float4 S[NR], next[NR];
    float value[NR], next_value[NR];
    auto ask = [&](float4 (&rows)[NR], float (&values)[NR], int first) __attribute__((always_inline)) {
#pragma unroll
      for (int r = 0; r < NR; ++r) {      // always a valid address; what is past the end is not used
        const int v = min(first + group + r * R, V - 1);
        rows[r] = load_four(kept + size_t(v) * D);
        values[r] = to_float(row[a.v_off + h * V + v]);
      }
    };
    ask(S, value, 0);
    const float i = log_input_gate(to_float(row[a.i_off + h]), bias_i, a.cap);
    const float f = log_forget_gate(to_float(row[a.f_off + h]), bias_f, a.cap);
    const float4 q = in ? load_four(row + a.q_off + h * D + d0) : zero, k = in ? load_four(row + a.k_off + h * D + d0) : zero;
    const float top = fmaxf(f + m, i), keep = expf(f + m - top), take = expf(i - top);
    m = top;
    norm = make_float4(fmaf(keep, norm.x, take * k.x), fmaf(keep, norm.y, take * k.y), fmaf(keep, norm.z, take * k.z),
                       fmaf(keep, norm.w, take * k.w));
    float nq = dot4(norm, q);
    for (int off = lanes >> 1; off > 0; off >>= 1) nq += __shfl_xor(nq, off, 64);
    const float share = q_scale / (fmaxf(fabsf(nq * q_scale), expf(-m)) + kShareFloor);
    float* o_row = lds + ((t - start) & 1) * V;
    float squares = 0.f;
    for (int first = 0; first < V; first += R * NR) {
      const bool more = first + R * NR < V;
      if (more) ask(next, next_value, first + R * NR);
      float o[NR];
#pragma unroll
      for (int r = 0; r < NR; ++r) {
        const int v = first + group + r * R;
        const float tv = take * value[r];
        const float4 x = make_float4(fmaf(keep, S[r].x, tv * k.x), fmaf(keep, S[r].y, tv * k.y), fmaf(keep, S[r].z, tv * k.z),
                                     fmaf(keep, S[r].w, tv * k.w));
        o[r] = in ? dot4(x, q) : 0.f;
        if (in && v < V) *reinterpret_cast<float4*>(kept + size_t(v) * D) = x;
      }
      for (int off = lanes >> 1; off > 0; off >>= 1)
#pragma unroll
        for (int r = 0; r < NR; ++r) o[r] += __shfl_xor(o[r], off, 64);
      if (l == 0) {
#pragma unroll
        for (int r = 0; r < NR; ++r) {
          const int v = first + group + r * R;
          const float x = o[r] * share;
          if (v < V) { o_row[v] = x; squares = fmaf(x, x, squares); }
        }
      }
      if (more) {
#pragma unroll
        for (int r = 0; r < NR; ++r) { S[r] = next[r]; value[r] = next_value[r]; }
      }
    }
    squares = block_sum(squares, scratch);      // (its barriers also publish o_row)
    const float unit = 1.0f / sqrtf(squares / float(V) + a.eps);
    for (int v = threadIdx.x; v < V; v += threads)
      out[size_t(t) * a.out_stride + h * V + v] =
          from_float<T>(((o_row[v] * unit) * a.norm[h * V + v]) * sigmoid(to_float(row[a.gate_off + h * V + v])));
  }
  if (in && group == 0) *reinterpret_cast<float4*>(kept + size_t(V) * D) = norm;
  if (threadIdx.x == 0) a.maxima[size_t(slot) * a.heads + h] = m;
}

// Any sizes: the memory stays in memory, a wave a row (the normaliser is row vdim, with the value one).
template <typename T>
__global__ __launch_bounds__(256) void mlstm_general_kernel(MlstmArgs a) {
  extern __shared__ float lds[];      // q [dim], k [dim], o [vdim + 1]
  __shared__ float scratch[16];
  const int s = blockIdx.x, h = blockIdx.y, D = a.dim, V = a.vdim, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  float *qs = lds, *ks = lds + D, *os = lds + 2 * D;
  const int start = a.q_start[s], n = a.q_len[s], slot = a.state_slots[s];
  float* kept = a.memory + (size_t(slot) * a.heads + h) * size_t(V + 1) * D;
  float m = a.maxima[size_t(slot) * a.heads + h];
  const float q_scale = 1.0f / sqrtf(float(D)), bias_i = a.bias_i[h], bias_f = a.bias_f[h];
  T* out = (T*)a.out;
  for (int t = start; t < start + n; ++t) {
    const T* row = (const T*)a.proj + size_t(t) * a.stride;
    for (int d = threadIdx.x; d < D; d += 256) {
      qs[d] = to_float(row[a.q_off + h * D + d]) * q_scale;
      ks[d] = to_float(row[a.k_off + h * D + d]);
    }
    const float i = log_input_gate(to_float(row[a.i_off + h]), bias_i, a.cap);
    const float f = log_forget_gate(to_float(row[a.f_off + h]), bias_f, a.cap);
    const float top = fmaxf(f + m, i), keep = expf(f + m - top), take = expf(i - top);
    m = top;
    __syncthreads();
    for (int v = wave; v <= V; v += 4) {
      const float tv = v < V ? take * to_float(row[a.v_off + h * V + v]) : take;
      float* S = kept + size_t(v) * D;
      float o = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float x = fmaf(keep, S[d], tv * ks[d]);
        S[d] = x;
        o = fmaf(x, qs[d], o);
      }
      o = wave_sum(o);
      if (lane == 0) os[v] = o;
    }
    __syncthreads();
    const float share = 1.0f / (fmaxf(fabsf(os[V]), expf(-m)) + kShareFloor);
    float squares = 0.f;
    for (int v = threadIdx.x; v < V; v += 256) { const float x = os[v] * share; squares = fmaf(x, x, squares); }
    const float unit = 1.0f / sqrtf(block_sum(squares, scratch) / float(V) + a.eps);
    for (int v = threadIdx.x; v < V; v += 256)
      out[size_t(t) * a.out_stride + h * V + v] =
          from_float<T>((((os[v] * share) * unit) * a.norm[h * V + v]) * sigmoid(to_float(row[a.gate_off + h * V + v])));
    __syncthreads();
  }
  if (threadIdx.x == 0) a.maxima[size_t(slot) * a.heads + h] = m;
}

// ------------------------------------------------------------------------------------------ chunks
// Long portions in chunks of 64 tokens, three passes.  With a chunk's tokens 0 .. n-1, F_t the sum of the logarithms f_0 .. f_t,
// g_j = i_j - F_j and the memory (S0, n0, m0) before the chunk, x_t = max(m0, max_(j<=t) g_j) gives m_t = F_t + x_t and
//   S_t = exp(m0 - x_t) S0 + sum_(j<=t) exp(g_j - x_t) v_j k_j^T          (n likewise),
// every exponent at most zero.  (1) Every chunk's own sum against its own maximum M = F_last + max_j g_j, all side by side;
// (2) per memory number the chunks one after the other, which leaves in the sums' place what each chunk starts from; (3) every
// chunk's outputs.
//
// q, k and v are bfloat16, so every product of two of them is exact on the bfloat16 matrix instruction, which sums in float32.
// A float32 factor (weighted values, weighted scores, the memory) goes through it as three bfloat16 numbers that add up to
// its 24 bits: three instructions where the float32 instruction would take sixteen times as long as one.
constexpr int kMlstmChunk = 64;
constexpr int kChunkPitch = kMlstmChunk + 8;      // bfloat16 numbers of an LDS row of tokens: 16-byte pieces, rows on different banks
constexpr int kValueBlock = 64;                   // value numbers of a block of the first pass

struct MlstmScratch {
  float* sums;      // [chunk][heads][vdim + 1][dim]
  float* scalars;   // [chunk][heads][4]: F_last, M, m0
};

// What a lane's token of the chunk contributes, by one wave: F, g and the running maximum of g, float64.
template <typename T>
__device__ __forceinline__ void chunk_gates(const MlstmArgs& a, int h, int first, int len, double* F, double* g, double* gmax) {
  const int j = threadIdx.x & 63;
  const bool in = j < len;
  const T* row = (const T*)a.proj + size_t(first + (in ? j : 0)) * a.stride;
  const double i = log_input_gate(to_float(row[a.i_off + h]), a.bias_i[h], a.cap);
  double sum = in ? double(log_forget_gate(to_float(row[a.f_off + h]), a.bias_f[h], a.cap)) : 0.0;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double other = __shfl_up(sum, off, 64);
    if (j >= off) sum += other;
  }
  const double mine = in ? i - sum : -INFINITY;
  double top = mine;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double other = __shfl_up(top, off, 64);
    if (j >= off) top = fmax(top, other);
  }
  F[j] = sum;
  g[j] = mine;
  gmax[j] = top;
}

// x as three bfloat16 numbers (as bits) that add up to its 24 bits.
__device__ __forceinline__ void split3(float x, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
  hi = f32_to_bf16_bits(x);
  const float r = x - __uint_as_float(hi << 16);
  mid = f32_to_bf16_bits(r);
  lo = f32_to_bf16_bits(r - __uint_as_float(mid << 16));
}
// Two neighbours at once, packed.
__device__ __forceinline__ void split3_pair(float x, float y, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
  hi = pack_bf16x2(x, y);
  const float rx = x - __uint_as_float(hi << 16), ry = y - __uint_as_float(hi & 0xffff0000u);
  mid = pack_bf16x2(rx, ry);
  lo = pack_bf16x2(rx - __uint_as_float(mid << 16), ry - __uint_as_float(mid & 0xffff0000u));
}
__device__ __forceinline__ void split3_eight(const float4& x, const float4& y, bf16x8& hi, bf16x8& mid, bf16x8& lo) {
  uint4 h, m, l;
  split3_pair(x.x, x.y, h.x, m.x, l.x);
  split3_pair(x.z, x.w, h.y, m.y, l.y);
  split3_pair(y.x, y.y, h.z, m.z, l.z);
  split3_pair(y.z, y.w, h.w, m.w, l.w);
  hi = as_bf16x8(h);
  mid = as_bf16x8(m);
  lo = as_bf16x8(l);
}

// Columns 8 cg .. of the chunk's rows, transposed into LDS: dst[column][token], a thread two tokens and eight columns at a time.
// What is past the chunk's end or the last column is zero.  use(column, token pair, value of the first, of the second).
template <typename F>
__device__ __forceinline__ void each_pair(const bf16_t* src, long long stride, int len, int cols, F use) {
  const int p = threadIdx.x & 31;
  const uint4 none = make_uint4(0u, 0u, 0u, 0u);
  for (int cg = threadIdx.x >> 5; 8 * cg < cols; cg += blockDim.x >> 5) {
    const uint4 x = 2 * p < len ? ldg128(src + size_t(2 * p) * stride + 8 * cg) : none;
    const uint4 y = 2 * p + 1 < len ? ldg128(src + size_t(2 * p + 1) * stride + 8 * cg) : none;
    const uint32_t xs[4] = {x.x, x.y, x.z, x.w}, ys[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      use(8 * cg + 2 * c, p, xs[c] & 0xffffu, ys[c] & 0xffffu);
      use(8 * cg + 2 * c + 1, p, xs[c] >> 16, ys[c] >> 16);
    }
  }
}

__global__ __launch_bounds__(256) void mlstm_chunk_local_kernel(MlstmArgs a, MlstmScratch scratch, int n_seqs) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];      // weighted values [3][64][pitch], keys [dim][pitch]
  constexpr int C = kMlstmChunk, CP = kChunkPitch, VB = kValueBlock;
  __shared__ double F[C], g[C], gmax[C];
  __shared__ float weight[C];
  int s, ci;
  if (!chunk_of_block(a.q_start, a.q_len, n_seqs, C, blockIdx.x, s, ci)) return;
  const int h = blockIdx.y, v_begin = blockIdx.z * VB, D = a.dim, V = a.vdim;
  const int first = a.q_start[s] + ci * C, len = min(C, a.q_start[s] + a.q_len[s] - first);
  uint16_t* vt = reinterpret_cast<uint16_t*>(smem);
  uint16_t* kt = vt + 3 * VB * CP;
  const bf16_t* proj = (const bf16_t*)a.proj + size_t(first) * a.stride;
  if (threadIdx.x < 64) {
    chunk_gates<bf16_t>(a, h, first, len, F, g, gmax);
    weight[threadIdx.x] = int(threadIdx.x) < len ? expf(float(g[threadIdx.x] - gmax[C - 1])) : 0.f;
  }
  each_pair(proj + a.k_off + h * D, a.stride, len, D, [&](int d, int p, uint32_t x, uint32_t y) {
    reinterpret_cast<uint32_t*>(kt + d * CP)[p] = x | (y << 16);
  });
  __syncthreads();
  const int cols = min(VB, V - v_begin);
  each_pair(proj + a.v_off + h * V + v_begin, a.stride, len, cols, [&](int v, int p, uint32_t x, uint32_t y) {
    uint32_t hi, mid, lo;
    split3_pair(__uint_as_float(x << 16) * weight[2 * p], __uint_as_float(y << 16) * weight[2 * p + 1], hi, mid, lo);
    reinterpret_cast<uint32_t*>(vt + v * CP)[p] = hi;
    reinterpret_cast<uint32_t*>(vt + (VB + v) * CP)[p] = mid;
    reinterpret_cast<uint32_t*>(vt + (2 * VB + v) * CP)[p] = lo;
  });
  __syncthreads();
  const size_t number = size_t(blockIdx.x) * a.heads + h;      // the block's number is the chunk's row in the scratch
  float* U = scratch.sums + number * (size_t(V + 1) * D);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 31, hi = lane >> 5;
  const int tiles_d = (D + 31) / 32, tiles_v = (cols + 31) / 32;
  for (int tile = wave; tile < tiles_d * tiles_v; tile += 4) {
    const int v0 = (tile / tiles_d) * 32, d0 = (tile % tiles_d) * 32;
    const int vr = min(v0 + col, cols - 1), dr = min(d0 + col, D - 1);      // rows past the end are computed and not stored
    floatx16 acc = {0};
#pragma unroll
    for (int kk = 0; kk < C / 16; ++kk) {
      const int j = 16 * kk + 8 * hi;
      const bf16x8 key = as_bf16x8(*reinterpret_cast<const uint4*>(kt + dr * CP + j));
#pragma unroll
      for (int part = 0; part < 3; ++part)
        acc = mfma32(as_bf16x8(*reinterpret_cast<const uint4*>(vt + (part * VB + vr) * CP + j)), key, acc);
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int v = v0 + 8 * (r / 4) + 4 * hi + r % 4, d = d0 + col;
      if (v < cols && d < D) U[size_t(v_begin + v) * D + d] = acc[r];
    }
  }
  if (blockIdx.z == 0) {
    for (int d = threadIdx.x; d < D; d += 256) {
      float sum = 0.f;
      for (int j = 0; j < len; ++j) sum = fmaf(weight[j], to_float(bf16_t{kt[d * CP + j]}), sum);
      U[size_t(V) * D + d] = sum;
    }
    if (threadIdx.x == 0) {
      float* sc = scratch.scalars + 4 * number;
      sc[0] = float(F[C - 1]);
      sc[1] = float(F[C - 1] + gmax[C - 1]);
      if (ci == 0) sc[2] = a.maxima[size_t(a.state_slots[s]) * a.heads + h];      // (the next pass overwrites the slot's)
    }
  }
}

__global__ __launch_bounds__(256) void mlstm_chunk_carry_kernel(MlstmArgs a, MlstmScratch scratch) {
  constexpr int C = kMlstmChunk, AHEAD = 8;
  const int s = blockIdx.x, h = blockIdx.y, E = (a.vdim + 1) * a.dim, e = 4 * (blockIdx.z * 256 + threadIdx.x);
  const int n = a.q_len[s], slot = a.state_slots[s], used = (n + C - 1) / C;
  if (n <= 0) return;
  const bool live = e < E;
  const size_t number = size_t(a.q_start[s] / C + s) * a.heads + h;      // chunk ci: number + ci * heads
  float* at = scratch.sums + number * E + (live ? e : 0);
  float* sc = scratch.scalars + 4 * number;
  const size_t step = size_t(a.heads) * E, sc_step = size_t(4) * a.heads;
  float* kept = a.memory + (size_t(slot) * a.heads + h) * E + (live ? e : 0);
  float4 S = load_four(kept);
  float m = sc[2];
  for (int c0 = 0; c0 < used; c0 += AHEAD) {
    float4 U[AHEAD];
    float F[AHEAD], M[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const int ci = min(c0 + j, used - 1);
      U[j] = load_four(at + ci * step);
      F[j] = sc[ci * sc_step];
      M[j] = sc[ci * sc_step + 1];
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const int ci = c0 + j;
      if (ci < used) {
        if (live) *reinterpret_cast<float4*>(at + ci * step) = S;      // what the chunk starts from
        if (ci > 0 && blockIdx.z == 0 && threadIdx.x == 0) sc[ci * sc_step + 2] = m;
        const float top = fmaxf(F[j] + m, M[j]), keep = expf(F[j] + m - top), take = expf(M[j] - top);
        m = top;
        S = make_float4(fmaf(keep, S.x, take * U[j].x), fmaf(keep, S.y, take * U[j].y), fmaf(keep, S.z, take * U[j].z),
                        fmaf(keep, S.w, take * U[j].w));
      }
    }
  }
  if (live) *reinterpret_cast<float4*>(kept) = S;
  if (blockIdx.z == 0 && threadIdx.x == 0) a.maxima[size_t(slot) * a.heads + h] = m;
}

// The chunk's outputs: a block per (chunk, head), a wave NT columns of 32 value numbers for all 64 tokens.
template <int WAVES, int NT>
__global__ __launch_bounds__(64 * WAVES) void mlstm_chunk_apply_kernel(MlstmArgs a, MlstmScratch scratch, int n_seqs) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];      // weighted scores [3][64][pitch], values [vdim][pitch]
  constexpr int C = kMlstmChunk, CP = kChunkPitch;
  __shared__ double F[C], g[C], gmax[C];
  __shared__ float before[C], floor_of[C], own[2][C], past[WAVES][C], squares[WAVES][C], share[C], unit[C];
  int s, ci;
  if (!chunk_of_block(a.q_start, a.q_len, n_seqs, C, blockIdx.x, s, ci)) return;
  const int h = blockIdx.y, D = a.dim, V = a.vdim;
  const int first = a.q_start[s] + ci * C, len = min(C, a.q_start[s] + a.q_len[s] - first);
  uint16_t* ps = reinterpret_cast<uint16_t*>(smem);
  uint16_t* vt = ps + 3 * C * CP;
  const bf16_t* proj = (const bf16_t*)a.proj + size_t(first) * a.stride;
  const bf16_t *q = proj + a.q_off + h * D, *k = proj + a.k_off + h * D;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 31, hi = lane >> 5;
  const size_t number = size_t(blockIdx.x) * a.heads + h;
  const float* S0 = scratch.sums + number * (size_t(V + 1) * D);
  const float m0 = scratch.scalars[4 * number + 2], q_scale = 1.0f / sqrtf(float(D));
  if (wave == 0) {
    chunk_gates<bf16_t>(a, h, first, len, F, g, gmax);
    const double x = fmax(double(m0), gmax[lane]);
    before[lane] = expf(float(double(m0) - x));
    floor_of[lane] = expf(float(-(F[lane] + x)));
    own[1][lane] = 0.f;
  }
  each_pair(proj + a.v_off + h * V, a.stride, len, V, [&](int v, int p, uint32_t x, uint32_t y) {
    reinterpret_cast<uint32_t*>(vt + v * CP)[p] = x | (y << 16);
  });
  {
    // n0 . q: lane = token, the waves share the dimensions
    const bf16_t* row = q + size_t(min(lane, len - 1)) * a.stride;
    const float* n0 = S0 + size_t(V) * D;
    float sum = 0.f;
    for (int d = 8 * wave; d < D; d += 8 * WAVES)
      sum += dot4(load_four(n0 + d), load_four(row + d)) + dot4(load_four(n0 + d + 4), load_four(row + d + 4));
    past[wave][lane] = sum;
  }
  __syncthreads();
  if (wave < 3) {      // score tiles of 32 x 32: (0, 0), (1, 0), (1, 1); the fourth is all in the future
    const int ti = wave > 0, tj = wave == 2;
    const bf16_t* qr = q + size_t(min(32 * ti + col, len - 1)) * a.stride + 8 * hi;
    const bf16_t* kr = k + size_t(min(32 * tj + col, len - 1)) * a.stride + 8 * hi;
    floatx16 acc = {0};
#pragma unroll 8
    for (int d = 0; d < D; d += 16) acc = mfma32(as_bf16x8(ldg128(qr + d)), as_bf16x8(ldg128(kr + d)), acc);
    const int j = 32 * tj + col;
    const double gj = g[j];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = 32 * ti + 8 * (r / 4) + 4 * hi + r % 4;
      const float w = j <= i && i < len ? expf(float(gj - fmax(double(m0), gmax[i]))) : 0.f;
      const float p = j <= i && i < len ? (acc[r] * q_scale) * w : 0.f;
      uint32_t p0, p1, p2;
      split3(p, p0, p1, p2);
      ps[i * CP + j] = uint16_t(p0);
      ps[(C + i) * CP + j] = uint16_t(p1);
      ps[(2 * C + i) * CP + j] = uint16_t(p2);
      float sum = p;
#pragma unroll
      for (int off = 16; off > 0; off >>= 1) sum += __shfl_xor(sum, off, 64);
      if (col == 0) own[tj][i] = sum;
    }
  }
  __syncthreads();
  const int tiles_v = (V + 31) / 32;
  floatx16 o[NT][2];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    o[t][0] = floatx16{0};
    o[t][1] = floatx16{0};
    const int tile = wave + WAVES * t;
    if (tile >= tiles_v) continue;
    const int v = min(32 * tile + col, V - 1);
    const float* mem = S0 + size_t(v) * D + 8 * hi;
    const bf16_t* q0 = q + size_t(min(col, len - 1)) * a.stride + 8 * hi;
    const bf16_t* q1 = q + size_t(min(32 + col, len - 1)) * a.stride + 8 * hi;
#pragma unroll 4
    for (int d = 0; d < D; d += 16) {      // what the tokens before the chunk left
      bf16x8 b[3];
      split3_eight(load_four(mem + d), load_four(mem + d + 4), b[0], b[1], b[2]);
      const bf16x8 a0 = as_bf16x8(ldg128(q0 + d)), a1 = as_bf16x8(ldg128(q1 + d));
#pragma unroll
      for (int part = 2; part >= 0; --part) {
        o[t][0] = mfma32(a0, b[part], o[t][0]);
        o[t][1] = mfma32(a1, b[part], o[t][1]);
      }
    }
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int r = 0; r < 16; ++r) o[t][ti][r] *= q_scale * before[32 * ti + 8 * (r / 4) + 4 * hi + r % 4];
#pragma unroll
    for (int kk = 0; kk < C / 16; ++kk) {      // the chunk's own tokens; the first 32 see the first 32 only
      const int j = 16 * kk + 8 * hi;
      const bf16x8 value = as_bf16x8(*reinterpret_cast<const uint4*>(vt + v * CP + j));
#pragma unroll
      for (int part = 2; part >= 0; --part) {
        if (kk < 2) o[t][0] = mfma32(as_bf16x8(*reinterpret_cast<const uint4*>(ps + (part * C + col) * CP + j)), value, o[t][0]);
        o[t][1] = mfma32(as_bf16x8(*reinterpret_cast<const uint4*>(ps + (part * C + 32 + col) * CP + j)), value, o[t][1]);
      }
    }
  }
  if (threadIdx.x < C) {
    const int i = threadIdx.x;
    float nq = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) nq += past[w][i];
    nq = fmaf(nq * q_scale, before[i], own[0][i] + own[1][i]);
    share[i] = 1.0f / (fmaxf(fabsf(nq), floor_of[i]) + kShareFloor);
  }
  __syncthreads();
#pragma unroll
  for (int ti = 0; ti < 2; ++ti)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = 32 * ti + 8 * (r / 4) + 4 * hi + r % 4;
      float total = 0.f;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        o[t][ti][r] *= share[i];
        if (32 * (wave + WAVES * t) + col < V) total = fmaf(o[t][ti][r], o[t][ti][r], total);
      }
#pragma unroll
      for (int off = 16; off > 0; off >>= 1) total += __shfl_xor(total, off, 64);
      if (col == 0) squares[wave][i] = total;
    }
  __syncthreads();
  if (threadIdx.x < C) {
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) total += squares[w][threadIdx.x];
    unit[threadIdx.x] = 1.0f / sqrtf(total / float(V) + a.eps);
  }
  __syncthreads();
  bf16_t* out = (bf16_t*)a.out;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int v = 32 * (wave + WAVES * t) + col;
    if (v >= V) continue;
    const float w = a.norm[h * V + v];
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      float gate[16];
#pragma unroll
      for (int r = 0; r < 16; ++r)
        gate[r] = to_float(proj[size_t(min(32 * ti + 8 * (r / 4) + 4 * hi + r % 4, len - 1)) * a.stride + a.gate_off + h * V + v]);
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int i = 32 * ti + 8 * (r / 4) + 4 * hi + r % 4;
        if (i >= len) continue;
        out[size_t(first + i) * a.out_stride + h * V + v] = from_float<bf16_t>(((o[t][ti][r] * unit[i]) * w) * sigmoid(gate[r]));
      }
    }
  }
}

// ------------------------------------------------------------------------------------------ host side
constexpr int kMlstmLongPortion = 16;      // a step whose longest portion has more tokens takes the chunks

static bool mlstm_in_chunks(int dtype, int dim, int vdim) {
  return dtype == kBF16 && dim % 16 == 0 && dim <= 256 && vdim % 8 == 0 && vdim <= 512;
}
static size_t mlstm_local_lds(int dim) { return size_t(3 * kValueBlock + dim) * kChunkPitch * 2; }
static size_t mlstm_apply_lds(int vdim) { return size_t(3 * kMlstmChunk + vdim) * kChunkPitch * 2; }

// Lets a kernel ask for `bytes` of LDS, more than the 64 KB it gets unasked.
template <typename K>
static int allow_lds(K kernel, size_t bytes) {
  const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, int(bytes));
  if (e == hipSuccess) return 0;
  set_error("sp_mlstm: cannot raise the LDS limit: %s", hipGetErrorString(e));
  return 1;
}

static int launch_mlstm_chunks(hipStream_t s, const MlstmArgs& a, int T, int n_seqs, float* scratch) {
  const size_t rows = size_t(T / kMlstmChunk + n_seqs) * a.heads, E = size_t(a.vdim + 1) * a.dim;
  const MlstmScratch places = {scratch, scratch + rows * E};
  static bool raised = false;      // once, for the largest sizes the kernels take
  if (!raised) {
    if (allow_lds(mlstm_chunk_local_kernel, mlstm_local_lds(256)) || allow_lds(mlstm_chunk_apply_kernel<8, 1>, mlstm_apply_lds(256)) ||
        allow_lds(mlstm_chunk_apply_kernel<8, 2>, mlstm_apply_lds(512)))
      return 1;
    raised = true;
  }
  const dim3 chunks(T / kMlstmChunk + n_seqs, a.heads);      // a block per chunk number (chunk_of_block)
  mlstm_chunk_local_kernel<<<dim3(chunks.x, chunks.y, (a.vdim + kValueBlock - 1) / kValueBlock), 256, mlstm_local_lds(a.dim), s>>>(a, places, n_seqs);
  mlstm_chunk_carry_kernel<<<dim3(n_seqs, a.heads, unsigned((E / 4 + 255) / 256)), 256, 0, s>>>(a, places);
  const size_t lds = mlstm_apply_lds(a.vdim);
  if (a.vdim <= 128) mlstm_chunk_apply_kernel<4, 1><<<chunks, 256, lds, s>>>(a, places, n_seqs);
  else if (a.vdim <= 256) mlstm_chunk_apply_kernel<8, 1><<<chunks, 512, lds, s>>>(a, places, n_seqs);
  else mlstm_chunk_apply_kernel<8, 2><<<chunks, 512, lds, s>>>(a, places, n_seqs);
  return check_launch("sp_mlstm (chunks)");
}

// How a block of the step kernel holds a head's memory: lanes to a row, threads, rows a thread (0: no such kernel takes it; more
// than 8: it passes through the registers).
struct StepShape { int lanes, threads, rows; };
static StepShape mlstm_step_shape(int dim, int vdim) {
  StepShape shape = {1, 256, 0};
  if (dim % 4 || dim > 256) return shape;
  while (4 * shape.lanes < dim) shape.lanes *= 2;
  for (shape.threads = 256; shape.threads < 1024; shape.threads *= 2)
    if (vdim * shape.lanes <= 8 * shape.threads) break;
  const int R = shape.threads / shape.lanes, rows = (vdim + R - 1) / R;
  shape.rows = rows <= 1 ? 1 : rows <= 2 ? 2 : rows <= 4 ? 4 : rows <= 8 ? 8 : 16;
  return shape;
}

template <typename T>
static int launch_mlstm_step(hipStream_t s, const MlstmArgs& a, int n_seqs, StepShape shape) {
  const dim3 grid(n_seqs, a.heads);
  const size_t lds = size_t(2) * a.vdim * sizeof(float);
  switch (shape.rows) {
    case 1: mlstm_step_kernel<T, 1><<<grid, shape.threads, lds, s>>>(a, shape.lanes); break;
    case 2: mlstm_step_kernel<T, 2><<<grid, shape.threads, lds, s>>>(a, shape.lanes); break;
    case 4: mlstm_step_kernel<T, 4><<<grid, shape.threads, lds, s>>>(a, shape.lanes); break;
    case 8: mlstm_step_kernel<T, 8><<<grid, shape.threads, lds, s>>>(a, shape.lanes); break;
    default: mlstm_stream_kernel<T, 4><<<grid, shape.threads, lds, s>>>(a, shape.lanes); break;
  }
  return check_launch("sp_mlstm");
}

}  // namespace sprout

using namespace sprout;

extern "C" int sp_mlstm_takes(int dim, int vdim) { return dim > 0 && vdim > 0 && 2 * dim + vdim <= 15000; }

extern "C" long long sp_mlstm_scratch_floats(int dtype, int heads, int dim, int vdim, int n_seqs, int max_q_len, int T) {
  if (max_q_len <= kMlstmLongPortion || heads <= 0 || dim <= 0 || vdim <= 0 || !mlstm_in_chunks(dtype, dim, vdim)) return 0;
  return ((long long)T / kMlstmChunk + n_seqs) * heads * ((long long)(vdim + 1) * dim + 4);
}

extern "C" int sp_mlstm(void* stream, int dtype, const void* proj, long long stride, int q_off, int k_off, int v_off, int gate_off,
                        int i_off, int f_off, int heads, int dim, int vdim, float cap, const float* bias_i, const float* bias_f,
                        const float* norm, float eps, const int32_t* q_start, const int32_t* q_len, const int32_t* state_slots,
                        float* memory, float* maxima, void* out, long long out_stride, int T, int n_seqs, int max_q_len, float* scratch) {
  SP_REQUIRE(heads > 0 && sp_mlstm_takes(dim, vdim), "sp_mlstm: no kernel for heads of %d and %d numbers", dim, vdim);
  SP_REQUIRE(cap > 0.f, "sp_mlstm: the gates' cap must be positive, not %g", double(cap));
  const long long qk = (long long)heads * dim, vg = (long long)heads * vdim;
  SP_REQUIRE(T >= 0 && n_seqs >= 0 && q_off >= 0 && k_off >= 0 && v_off >= 0 && gate_off >= 0 && i_off >= 0 && f_off >= 0 &&
                 stride >= q_off + qk && stride >= k_off + qk && stride >= v_off + vg && stride >= gate_off + vg &&
                 stride >= i_off + heads && stride >= f_off + heads,
             "sp_mlstm: rows of %lld numbers do not hold q, k, v and the gates", stride);
  SP_REQUIRE(out_stride >= vg, "sp_mlstm: a row of %lld results does not hold the heads' outputs", out_stride);
  SP_REQUIRE(proj && bias_i && bias_f && norm && q_start && q_len && state_slots && memory && maxima && out, "sp_mlstm: null operand");
  SP_REQUIRE(dtype == kF32 || dtype == kBF16, "sp_mlstm: unsupported dtype %d", dtype);
  SP_REQUIRE(heads <= 65535, "sp_mlstm: %d heads are more than a launch's second dimension holds", heads);
  if (T == 0 || n_seqs == 0) return 0;
  const MlstmArgs a = {proj, stride, q_off, k_off, v_off, gate_off, i_off, f_off, heads, dim, vdim, cap, bias_i, bias_f, norm, eps,
                       q_start, q_len, state_slots, memory, maxima, out, out_stride};
  hipStream_t s = (hipStream_t)stream;
  // whether rows of q, k and v (and the memory's) start at whole pieces of `numbers` numbers
  auto rows_at = [&](int numbers) {
    return stride % numbers == 0 && q_off % numbers == 0 && k_off % numbers == 0 && v_off % numbers == 0 && dim % numbers == 0 &&
           (reinterpret_cast<uintptr_t>(proj) % 16) == 0 && (reinterpret_cast<uintptr_t>(memory) % 16) == 0;
  };
  if (scratch && sp_mlstm_scratch_floats(dtype, heads, dim, vdim, n_seqs, max_q_len, T) > 0 && rows_at(8) &&
      (reinterpret_cast<uintptr_t>(scratch) % 16) == 0)
    return launch_mlstm_chunks(s, a, T, n_seqs, scratch);
  const StepShape shape = mlstm_step_shape(dim, vdim);
  if (shape.rows && rows_at(4)) return dtype == kF32 ? launch_mlstm_step<float>(s, a, n_seqs, shape) : launch_mlstm_step<bf16_t>(s, a, n_seqs, shape);
  const size_t lds = size_t(2 * dim + vdim + 1) * sizeof(float);
  const dim3 grid(n_seqs, heads);
  if (dtype == kF32) mlstm_general_kernel<float><<<grid, 256, lds, s>>>(a);
  else mlstm_general_kernel<bf16_t><<<grid, 256, lds, s>>>(a);
  return check_launch("sp_mlstm (memory in memory)");
}
