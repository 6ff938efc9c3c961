// Shared device helpers for the gfx950 kernels: element types, conversions,
// wave64 reductions, and the error convention of the C entry points.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

typedef __bf16 bf16_t;

#define GL3_WAVE 64

// ---- error convention: every entry point returns 0 or a negative code and
// leaves a message that gl3_last_error() returns.
extern "C" const char* gl3_last_error();
void gl3_set_error(const char* fmt, ...);

#define GL3_REQUIRE(cond, ...)            \
  do {                                    \
    if (!(cond)) {                        \
      gl3_set_error(__VA_ARGS__);         \
      return -1;                          \
    }                                     \
  } while (0)

#define GL3_LAUNCH_CHECK()                                              \
  do {                                                                  \
    hipError_t e__ = hipGetLastError();                                 \
    if (e__ != hipSuccess) {                                            \
      gl3_set_error("%s: launch failed: %s", __func__, hipGetErrorString(e__)); \
      return -2;                                                        \
    }                                                                   \
  } while (0)

// dtype codes shared with the Python side
enum { GL3_F32 = 0, GL3_BF16 = 1 };

template <typename T> __device__ __forceinline__ float to_f32(T v);
template <> __device__ __forceinline__ float to_f32<float>(float v) { return v; }
template <> __device__ __forceinline__ float to_f32<bf16_t>(bf16_t v) { return static_cast<float>(v); }

template <typename T> __device__ __forceinline__ T from_f32(float v);
template <> __device__ __forceinline__ float from_f32<float>(float v) { return v; }
template <> __device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) { return static_cast<bf16_t>(v); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ double wave_sum_f64(double v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}

// Sum over a block of up to 1024 threads; every thread gets the result.
// `scratch` holds at least 16 floats of shared memory. The order of the sum
// depends only on the block size.
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  v = wave_sum(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += scratch[i];
  return t;
}
__device__ __forceinline__ double block_sum_f64(double v, double* scratch) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  v = wave_sum_f64(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  double t = 0.0;
  for (int i = 0; i < nw; ++i) t += scratch[i];
  return t;
}
__device__ __forceinline__ float block_max(float v, float* scratch) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  v = wave_max(v);
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  float t = scratch[0];
  for (int i = 1; i < nw; ++i) t = fmaxf(t, scratch[i]);
  return t;
}

// ---- what a product's epilogue may apply besides its own rule: a bias per output column (float;
// for the gated epilogue the gate's biases, then the up's), and the activation of the gated
// epilogue. The reference's feed-forward is silu without biases (J/inference/InferenceCore.java:158-166).
// How one kv head's keys and values lie inside a page of the cache. A key page holds
// [position][head_dim] elements, a value page [head_dim][position] (transposed), but not row by
// row: in tiles of 16 rows x 8 columns (16 bytes of bfloat16 a row), the tiles of the same 16 rows
// one after another along the columns. A matrix-core operand (lane r, q: row r, the 8 elements at
// column block q) of 16 rows x 32 columns is then 1 KB of consecutive memory in lane order, where
// rows lying one after another would make every lane touch a line of its own, which costs a CU's
// first-level cache four times the time.
//   values: tile (dim / 16, position / 8), row dim % 16, element position % 8
//   keys:   32 positions make two tiles: the positions with bit 2 clear, then those with it set, so
//           row i of the first is position 8 * (i / 4) + i % 4 of the 32 and row i of the second the
//           position 4 further. (The decode kernel's two score tiles of a chunk of 32 keys: a lane
//           then holds the probabilities of 8 consecutive keys, one 16-byte load of a value row.)
// page_size is a multiple of 32, head_dim of 16; 32 positions of a key page are still 32 * head_dim
// consecutive elements, and 8 elements that are consecutive along a row stay consecutive.
__device__ __forceinline__ long gl3_k_offset(int position_in_page, int dim, int head_dim) {
  const int p = position_in_page;
  const int tile = (p >> 5) * 2 + ((p >> 2) & 1), row = ((p >> 3) & 3) * 4 + (p & 3);
  return ((long)(tile * (head_dim >> 3) + (dim >> 3)) << 7) + (row << 3) + (dim & 7);
}
__device__ __forceinline__ long gl3_v_offset(int dim, int position_in_page, int page_size) {
  return ((long)((dim >> 4) * (page_size >> 3) + (position_in_page >> 3)) << 7) + ((dim & 15) << 3) + (position_in_page & 7);
}

// Element (row n, column k) of a matrix that is kept in the order of the matrix operands:
// [strip of 16 rows][k-step of 32][lane = 16 * (k block of 8) + row][8 elements], `steps` k-steps a strip
// (lib.tile_weight; 8 consecutive k of a row lie together).
__host__ __device__ __forceinline__ long gl3_operand_offset(long n, int k, int steps) {
  return (((n >> 4) * steps + (k >> 5)) << 9) + (((k & 31) >> 3) << 7) + ((n & 15) << 3) + (k & 7);
}
// The same for the packed strips of 8 rows: [strip of 8 rows][step of 64 k][lane = 16 * (k block of 8 inside its
// half) + 8 * (half of the step) + row][8 elements], `steps` steps of 64 a strip (lib.tile_weight8).
__host__ __device__ __forceinline__ long gl3_packed_offset(long n, int k, int steps) {
  return (((n >> 3) * steps + (k >> 6)) << 9) + (((k & 31) >> 3) << 7) + (((k >> 5) & 1) << 6) + ((n & 7) << 3) + (k & 7);
}
// Where element (n, k) of W lies. order 0: rows as stored (ldw); 1: the operands' order; 2: the packed strips of 8.
// `pos` (order 1, may be null): the place of each row in a copy whose strips hold the rows in another order.
__host__ __device__ __forceinline__ long gl3_w_offset(int order, long n, int k, long ldw, int steps, const int* pos) {
  if (order == 0) return n * ldw + k;
  if (order == 1) return gl3_operand_offset(pos ? pos[n] : n, k, steps);
  return gl3_packed_offset(n, k, steps);
}

enum { GL3_ACT_SILU = 0, GL3_ACT_GELU_TANH = 1, GL3_ACT_QUICK_GELU = 2 };
#define GL3_ACT_KNOWN(act) ((act) >= GL3_ACT_SILU && (act) <= GL3_ACT_QUICK_GELU)

template <bool FAST>
__device__ __forceinline__ float gl3_activation(float v, int act) {
  if (act == GL3_ACT_GELU_TANH) {
    // 0.5 v (1 + tanh(sqrt(2/pi) (v + 0.044715 v^3))) = v / (1 + exp(-2 u))
    const float u = 0.7978845608028654f * (v + 0.044715f * v * v * v);
    return v / (1.0f + (FAST ? __expf(-2.0f * u) : expf(-2.0f * u)));
  }
  if (act == GL3_ACT_QUICK_GELU) {   // v * sigmoid(1.702 v), the sigmoid form of gelu
    const float u = 1.702f * v;
    return v / (1.0f + (FAST ? __expf(-u) : expf(-u)));
  }
  return v / (1.0f + (FAST ? __expf(-v) : expf(-v)));
}

// What a description may do to attention scores and outputs beyond the plain rule (``lib.ScoreRule``): the query at
// position p counts `1 + temp_coef ln(floor((p + 1) / temp_every) + 1)` times (temp_every 0: once); a score is bounded
// to `softcap * tanh(score / softcap)` (softcap 0: not) before any bias that grows with the distance is taken off; and
// the heads' outputs are multiplied by sigmoid of the gate rows' elements (gate null: not), row t at gate + t gate_ld,
// the elements in the order of the output's.
struct Gl3ScoreRule {
  float softcap;
  float temp_coef;
  int temp_every;
  const void* gate;
  long gate_ld;
  bool any() const { return softcap != 0.f || temp_every != 0 || gate != nullptr; }
};
#define GL3_CHECK_RULE(r, who)                                                                                       \
  GL3_REQUIRE((r).softcap >= 0.f && (r).temp_every >= 0, who ": a soft cap of %g, a temperature that steps every %d", \
              (double)(r).softcap, (r).temp_every)
__device__ __forceinline__ float gl3_query_temperature(int p, const Gl3ScoreRule& r) {
  return r.temp_every > 0 ? 1.0f + r.temp_coef * logf((float)((p + 1) / r.temp_every + 1)) : 1.0f;
}
// tanh by one exponential and one reciprocal: 1 - 2 / (1 + e^(2y)), given y2 = 2 y log2(e); its error is one of
// 32-bit rounding of numbers around one (not relative to a small tanh). gl3_tanh_part: 1 / (1 + e^(2y)) alone.
__device__ __forceinline__ float gl3_tanh_part(float y2) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(y2)); }
__device__ __forceinline__ float gl3_tanh_of_exponent(float y2) { return fmaf(-2.0f, gl3_tanh_part(y2), 1.0f); }
__device__ __forceinline__ float gl3_sigmoid_fast(float z) {
  return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

// The gated epilogue's rule in full: act(gate) * (up + shift), where a positive `limit` first bounds the
// gate from above (min(gate, limit)) and the up value on both sides (clamp(up, -limit, limit)). The
// reference's feed-forward is limit = 0 (none), shift = 0.
template <bool FAST>
__device__ __forceinline__ float gl3_gated(float gate, float up, int act, float limit, float shift) {
  if (limit > 0.f) {
    gate = fminf(gate, limit);
    up = fminf(fmaxf(up, -limit), limit);
  }
  return gl3_activation<FAST>(gate, act) * (up + shift);
}
