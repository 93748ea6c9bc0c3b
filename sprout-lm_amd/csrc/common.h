// Shared helpers of the HIP kernels: storage types, conversions, reductions, error reporting.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdio.h>

namespace sprout {

// Element type codes of the C interface.
enum DType : int { kF32 = 0, kBF16 = 1 };

struct bf16_t { uint16_t bits; };

__device__ __forceinline__ float to_float(float v) { return v; }
__device__ __forceinline__ float to_float(bf16_t v) { return __uint_as_float(uint32_t(v.bits) << 16); }

// Round to nearest even; NaN stays NaN.  gfx950 converts in hardware (v_cvt_pk_bf16_f32).
__device__ __forceinline__ uint16_t f32_to_bf16_bits(float f) {
  return __builtin_bit_cast(uint16_t, static_cast<__bf16>(f));
}
template <typename T> __device__ __forceinline__ T from_float(float f);
template <> __device__ __forceinline__ float from_float<float>(float f) { return f; }
template <> __device__ __forceinline__ bf16_t from_float<bf16_t>(float f) { return bf16_t{f32_to_bf16_bits(f)}; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}

// Sum over a block of up to 1024 threads; every thread gets the result. `scratch` holds 16 floats.
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  v = wave_sum(v);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = (blockDim.x + 63) >> 6;
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float total = 0.f;
  for (int w = 0; w < waves; ++w) total += scratch[w];
  return total;
}

// Activations of a gated product, numbered as in the C interface: 0 = SiLU(g) * u; 1 = the clamped form
// g' = min(g, limit), u' = clamp(u, -limit, limit), g' * sigmoid(1.702 g') * (u' + 1); 2 = max(g, 0) * u;
// 3 = gelu(g) * u with the tanh form of gelu.
enum GateAct : int { kActSilu = 0, kActClampedSwish = 1, kActRelu = 2, kActGeluTanh = 3, kGateActs = 4 };
constexpr float kSwishSlope = 1.702f;
// The tanh form of gelu: 0.5 z (1 + tanh(y)) = z / (1 + exp(-2 y)), y = sqrt(2 / pi) (z + 0.044715 z^3).
__device__ __forceinline__ float gelu_tanh_exponent(float z) { return -1.5957691216057308f * (z + 0.044715f * z * z * z); }
__device__ __forceinline__ float gelu_tanh(float z) { return z / (1.0f + expf(gelu_tanh_exponent(z))); }
__device__ __forceinline__ float gated_value(float g, float u, int act, float limit) {
  if (act == kActClampedSwish) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.0f + expf(-kSwishSlope * g)) * (u + 1.0f);
  }
  if (act == kActRelu) return fmaxf(g, 0.f) * u;
  if (act == kActGeluTanh) return gelu_tanh(g) * u;
  return g / (1.0f + expf(-g)) * u;
}

// What a plain product's epilogue does to a number before it is stored: 0 = nothing, 1 = the square of max(x, 0).
enum StoreAct : int { kStoreAsIs = 0, kStoreReluSquared = 1 };
__device__ __forceinline__ float stored_value(float v, int act) {
  if (act == kStoreReluSquared) { v = fmaxf(v, 0.f); v *= v; }
  return v;
}

// Which earlier keys a query sees, and what stands between q . k and a key's weight.
struct ScoreStage {
  int window;          // > 0: keys with position - key < window
  int chunk;           // > 0: only keys of the query's own block of `chunk` positions, counted from position 0
  float cap;           // > 0: the scaled score s becomes cap * tanh(s / cap)
  const float* sinks;  // one number per query head whose exponential joins the softmax's denominator (null: none)
  int keep;            // > 0: the sequence's first `keep` keys stay visible to every later query, whatever the window
  const float* bias;   // one number per query head: a visible key's weight is sigmoid(score + bias), not normalised over
                       // the keys, in place of the softmax (null: the softmax)
  const void* gate;    // head h's output of token t is multiplied by sigmoid(gate[t * gate_stride + h]), numbers of the
  long long gate_stride;  // storage type (null: none)
};
template <typename T>
__device__ __forceinline__ float head_gate_of(const ScoreStage& st, size_t token, int head) {
  return st.gate ? 1.0f / (1.0f + expf(-to_float(((const T*)st.gate)[token * st.gate_stride + head]))) : 1.f;
}
// The first key that a query at `pos` sees.
__device__ __forceinline__ int first_visible(int pos, int window, int chunk) {
  int lo = window > 0 ? max(0, pos - window + 1) : 0;
  if (chunk > 0) lo = max(lo, pos - pos % chunk);
  return lo;
}

// Error text of the last failed call on this thread.
void set_error(const char* fmt, ...);
int check_launch(const char* what);

}  // namespace sprout

#define SP_REQUIRE(cond, ...)                 \
  do {                                        \
    if (!(cond)) {                            \
      sprout::set_error(__VA_ARGS__);         \
      return 1;                               \
    }                                         \
  } while (0)
