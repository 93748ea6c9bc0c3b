// Attention over a latent: what stands between the projections and the attention kernel.
//
// The cache holds per token the key [latent, rotated part, zeros up to `width`] of one key/value head and as value the
// latent in the same width (the value pool's columns behind the latent are never written and stay zero), so that every
// attention kernel for one key/value head and heads of `width` takes it.  Queries for that attention are
// [query . U_k (rank numbers, written by the per-head product), rotated part, zeros].  Up to three jobs a launch, a block a
// token and job: norm the latent, turn the shared key part and cache both; turn every head's query part; norm a query latent.
//
// Rotation: the first rot_dims numbers of a rotated part turn, (2i, 2i + 1) or (i, i + rot_dims / 2) together, by
// position * freq[i], and cosine and sine are multiplied by `magnitude`; the rest pass unchanged.  exact != 0: angle, sine
// and cosine in float64 (the float32 path), else float32.
#include "common.h"
#include "sprout_hip.h"

namespace sprout {

struct LatentArgs {
  int heads, dim, rot, rank, width;
  float eps;
  const int32_t* positions;
  const double* freq;
  int rot_dims;
  float magnitude;
  int halves, exact;
  const void* kv;              // rows with the latent and the shared key part (null: no such job)
  int kv_stride, kv_off;
  const void* kv_norm;
  const int32_t* slot_mapping;
  void *k_pool, *v_pool;
  int page_size;
  const void* q;               // rows with the heads' queries (null: no such job)
  int q_stride, q_off;
  void* q_out;
  const void* cq;              // rows with a query latent (null: no such job)
  int cq_stride, cq_off, cq_rank;
  const void* cq_norm;
  void* cq_out;
  int jobs[3];                 // blockIdx.y: which job (0 the latent, 1 the queries, 2 the query latent)
};

// One over the root mean square of n numbers, over the whole block.
template <typename T>
__device__ __forceinline__ float unit_of(const T* x, int n, float eps, float* scratch) {
  float sum = 0.f;
  for (int d = threadIdx.x; d < n; d += blockDim.x) {
    const float v = to_float(x[d]);
    sum = fmaf(v, v, sum);
  }
  return 1.0f / sqrtf(block_sum(sum, scratch) / float(n) + eps);
}

template <typename T, typename TW>
__global__ __launch_bounds__(256) void latent_prepare_kernel(LatentArgs a) {
  extern __shared__ float cs[];      // [rot_dims / 2][2] cosine, sine (times magnitude)
  __shared__ float scratch[16];
  const int t = blockIdx.x, rank = a.rank, rot = a.rot, width = a.width, pairs = a.rot_dims / 2;
  const int job = a.jobs[blockIdx.y];
  if (job < 2 && a.rot_dims > 0) {
    const int pos = a.positions[t];
    for (int i = threadIdx.x; i < pairs; i += blockDim.x) {
      float c, s;
      if (a.exact) {
        const double angle = double(pos) * a.freq[i];
        c = float(cos(angle) * double(a.magnitude));
        s = float(sin(angle) * double(a.magnitude));
      } else {
        const float angle = float(pos) * float(a.freq[i]);
        c = cosf(angle) * a.magnitude;
        s = sinf(angle) * a.magnitude;
      }
      cs[2 * i] = c;
      cs[2 * i + 1] = s;
    }
    __syncthreads();
  }
  auto turned = [&](const T* part, int d) -> float {
    if (d >= a.rot_dims) return to_float(part[d]);
    int i, at_u, at_v;
    bool second;
    if (a.halves) {
      second = d >= pairs;
      i = second ? d - pairs : d;
      at_u = i;
      at_v = i + pairs;
    } else {
      second = d & 1;
      i = d >> 1;
      at_u = 2 * i;
      at_v = 2 * i + 1;
    }
    const float u = to_float(part[at_u]), v = to_float(part[at_v]), c = cs[2 * i], s = cs[2 * i + 1];
    return second ? v * c + u * s : u * c - v * s;
  };

  if (job == 0) {
    const T* row = (const T*)a.kv + size_t(t) * a.kv_stride + a.kv_off;
    const TW* norm_w = (const TW*)a.kv_norm;
    const int slot = a.slot_mapping[t];
    if (slot >= 0) {      // the same in every thread
      const float scale = unit_of(row, rank, a.eps, scratch);
      const int page = slot / a.page_size, off = slot - page * a.page_size;
      T* key = (T*)a.k_pool + (size_t(page) * a.page_size + off) * width;
      T* value = (T*)a.v_pool + size_t(page) * width * a.page_size + off;      // [page][dim][token]
      for (int d = threadIdx.x; d < rank; d += blockDim.x) {
        const T c = from_float<T>((to_float(row[d]) * scale) * to_float(norm_w[d]));
        key[d] = c;
        value[size_t(d) * a.page_size] = c;
      }
      for (int d = threadIdx.x; d < width - rank; d += blockDim.x) key[rank + d] = from_float<T>(d < rot ? turned(row + rank, d) : 0.f);
    }
  }
  if (job == 2) {
    const T* row = (const T*)a.cq + size_t(t) * a.cq_stride + a.cq_off;
    const TW* norm_w = (const TW*)a.cq_norm;
    const float scale = unit_of(row, a.cq_rank, a.eps, scratch);
    T* out = (T*)a.cq_out + size_t(t) * a.cq_rank;
    for (int d = threadIdx.x; d < a.cq_rank; d += blockDim.x) out[d] = from_float<T>((to_float(row[d]) * scale) * to_float(norm_w[d]));
  }
  if (job == 1) {
    const T* row = (const T*)a.q + size_t(t) * a.q_stride + a.q_off;
    T* out = (T*)a.q_out + size_t(t) * a.heads * width;
    const int tail = width - rank;
    for (int j = threadIdx.x; j < a.heads * tail; j += blockDim.x) {
      const int h = j / tail, d = j - h * tail;
      out[h * width + rank + d] = from_float<T>(d < rot ? turned(row + h * (a.dim + rot) + a.dim, d) : 0.f);
    }
  }
}

}  // namespace sprout

using namespace sprout;

extern "C" int sp_latent_prepare(void* stream, int dtype, int heads, int dim, int rot, int rank, int width, int norm_w_dtype,
                                 float eps, const int32_t* positions, const double* freq, int rot_dims, float magnitude,
                                 int pairing, int exact, const void* kv, int kv_stride, int kv_off, const void* kv_norm,
                                 const int32_t* slot_mapping, void* k_pool, void* v_pool, int page_size, int num_pages,
                                 const void* q, int q_stride, int q_off, void* q_out, const void* cq, int cq_stride, int cq_off,
                                 int cq_rank, const void* cq_norm, void* cq_out, int T) {
  SP_REQUIRE(T >= 0 && heads > 0 && dim >= 0 && rot >= 0 && rank > 0 && width >= rank + rot, "sp_latent_prepare: bad sizes");
  SP_REQUIRE(rot_dims >= 0 && rot_dims <= rot && rot_dims % 2 == 0, "sp_latent_prepare: %d of %d numbers turn", rot_dims, rot);
  SP_REQUIRE(pairing == 0 || pairing == 1, "sp_latent_prepare: no pairing %d", pairing);
  SP_REQUIRE(positions && (rot_dims == 0 || freq), "sp_latent_prepare: null operand");
  SP_REQUIRE(!kv || (kv_off >= 0 && kv_stride >= kv_off + rank + rot && kv_norm && slot_mapping && k_pool && v_pool &&
                     page_size > 0 && num_pages > 0),
             "sp_latent_prepare: a row of %d numbers does not hold the latent, or there are no pools to write to", kv_stride);
  SP_REQUIRE(!q || (q_off >= 0 && q_stride >= q_off + heads * (dim + rot) && q_out),
             "sp_latent_prepare: a row of %d numbers does not hold the queries", q_stride);
  SP_REQUIRE(!cq || (cq_off >= 0 && cq_rank > 0 && cq_stride >= cq_off + cq_rank && cq_norm && cq_out),
             "sp_latent_prepare: a row of %d numbers does not hold the query latent", cq_stride);
  SP_REQUIRE((dtype == kF32 || dtype == kBF16) && (norm_w_dtype == kF32 || norm_w_dtype == kBF16),
             "sp_latent_prepare: unsupported dtypes %d, %d", dtype, norm_w_dtype);
  if (T == 0 || (!kv && !q && !cq)) return 0;
  hipStream_t s = (hipStream_t)stream;
  LatentArgs a = {heads, dim, rot, rank, width, eps, positions, freq, rot_dims, magnitude, pairing, exact, kv, kv_stride, kv_off,
                        kv_norm, slot_mapping, k_pool, v_pool, page_size, q, q_stride, q_off, q_out, cq, cq_stride, cq_off, cq_rank,
                        cq_norm, cq_out, {0, 0, 0}};
  int n_jobs = 0;
  if (kv) a.jobs[n_jobs++] = 0;
  if (q) a.jobs[n_jobs++] = 1;
  if (cq) a.jobs[n_jobs++] = 2;
  const dim3 grid(T, n_jobs);
  const size_t lds = size_t(rot_dims > 0 ? rot_dims : 2) * sizeof(float);
  if (dtype == kF32 && norm_w_dtype == kF32) latent_prepare_kernel<float, float><<<grid, 256, lds, s>>>(a);
  else if (dtype == kF32) latent_prepare_kernel<float, bf16_t><<<grid, 256, lds, s>>>(a);
  else if (norm_w_dtype == kF32) latent_prepare_kernel<bf16_t, float><<<grid, 256, lds, s>>>(a);
  else latent_prepare_kernel<bf16_t, bf16_t><<<grid, 256, lds, s>>>(a);
  return check_launch("sp_latent_prepare");
}
