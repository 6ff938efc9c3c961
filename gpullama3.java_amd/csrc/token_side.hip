// What a token's own row of a side table adds behind a layer's sublayers:
//   x += w * unit(W_proj g),   g = act(W_gate x) * e,   unit(y) = y over its root mean square (eps inside the root)
// x: the 32-bit residual row itself, e: the layer's columns of the token's row. Two kernels; the product with W_proj stands
// between them.
//   gl3_side_gate      g in the activations' type, padded with zeros to whole steps of the next product
//   gl3_norm_add_next  the norm and the sum, and with the completed row what the norm that reads it next would make of it
#include "common.h"

typedef __bf16 ts_bf16x8 __attribute__((ext_vector_type(8)));
typedef float ts_f32x4 __attribute__((ext_vector_type(4)));

struct SideGate {
  int d, dim, T, act;
  long lde, ldg;        // floats a row of the table and of g
  int col_e, dim_pad;
};
template <typename TE>
__device__ __forceinline__ float side_value(float v, int t, int n, const SideGate& s, const int* __restrict__ ids, const TE* __restrict__ table) {
  if (n >= s.dim) return 0.f;
  return gl3_activation<false>(v, s.act) * to_f32<TE>(table[(long)ids[t] * s.lde + s.col_e + n]);
}

// On the matrix cores, from the 32-bit rows (rounded to bfloat16 on their way into the operand): a block takes 16 tokens x
// 16 NT rows of W_gate, its NW waves share out K in runs of four steps of 32, asked for together, and their sums are added up
// in wave order. d must be a multiple of 8. (Rows and columns that do not exist read others' numbers and are not stored.)
template <int NT, int NW>
__global__ __launch_bounds__(NW * 64) void side_gate_mfma_kernel(const float* __restrict__ x, const bf16_t* __restrict__ w,
                                                                 const bf16_t* __restrict__ table, const int* __restrict__ ids,
                                                                 bf16_t* __restrict__ g, SideGate s) {
  __shared__ float part[NW][NT][16][17];
  const int t0 = blockIdx.x * 16, n0 = blockIdx.y * 16 * NT;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, li = lane & 15, lq = lane >> 4;
  const float* xp = x + (long)(t0 + li < s.T ? t0 + li : 0) * s.d;
  const bf16_t* wp[NT];
  ts_f32x4 acc[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    const int n = n0 + 16 * nt + li;
    wp[nt] = w + (long)(n < s.dim ? n : 0) * s.d;
    acc[nt] = ts_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const ts_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int k0 = 128 * wave; k0 < s.d; k0 += 128 * NW) {
    ts_f32x4 lo[4], hi[4];
    ts_bf16x8 b[4][NT];
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      const int k = k0 + 32 * st + 8 * lq, at = k < s.d ? k : 0;
      lo[st] = *reinterpret_cast<const ts_f32x4*>(xp + at);
      hi[st] = *reinterpret_cast<const ts_f32x4*>(xp + at + 4);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) b[st][nt] = *reinterpret_cast<const ts_bf16x8*>(wp[nt] + at);
    }
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      ts_bf16x8 a;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        a[e] = static_cast<bf16_t>(lo[st][e]);
        a[4 + e] = static_cast<bf16_t>(hi[st][e]);
      }
      if (k0 + 32 * st + 8 * lq >= s.d) a = zero;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const ts_bf16x8 bb = k0 + 32 * st + 8 * lq < s.d ? b[st][nt] : zero;
        acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bb, acc[nt], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][nt][4 * lq + i][li] = acc[nt][i];
  __syncthreads();
  for (int i = threadIdx.x; i < NT * 256; i += NW * 64) {
    const int r = i / (16 * NT), c = i % (16 * NT), n = n0 + c, t = t0 + r;
    if (t >= s.T || n >= s.dim_pad) continue;
    float v = 0.f;
#pragma unroll
    for (int wv = 0; wv < NW; ++wv) v += part[wv][c >> 4][r][c & 15];
    g[(long)t * s.ldg + n] = static_cast<bf16_t>(side_value<bf16_t>(v, t, n, s, ids, table));
  }
}

// Any sizes and types: a wave a (token, row of W_gate).
template <typename TW>
__global__ __launch_bounds__(256) void side_gate_kernel(const float* __restrict__ x, const TW* __restrict__ w, const TW* __restrict__ table,
                                                        const int* __restrict__ ids, TW* __restrict__ g, SideGate s) {
  const int t = blockIdx.x, n = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (n >= s.dim_pad) return;
  float v = 0.f;
  if (n < s.dim)
    for (int k = lane; k < s.d; k += 64) v = fmaf(to_f32<TW>(from_f32<TW>(x[(long)t * s.d + k])), to_f32<TW>(w[(long)n * s.d + k]), v);
  v = wave_sum(v);
  if (lane == 0) g[(long)t * s.ldg + n] = from_f32<TW>(side_value<TW>(v, t, n, s, ids, table));
}

extern "C" int gl3_side_gate(const float* x, const void* w, int dtype, const void* table, long lde, int col_e, const int* ids,
                             void* g, long ldg, int dim_pad, int T, int d, int dim, int act, int mfma, hipStream_t stream) {
  if (T == 0) return 0;
  GL3_REQUIRE(x && w && table && ids && g && T > 0 && d > 0 && dim > 0, "gl3_side_gate: bad arguments");
  GL3_REQUIRE(col_e >= 0 && col_e + (long)dim <= lde && dim_pad >= dim && dim_pad <= ldg && GL3_ACT_KNOWN(act),
              "gl3_side_gate: columns %d .. of rows of %ld, %d of %d columns of rows of %ld", col_e, lde, dim, dim_pad, ldg);
  const SideGate s{d, dim, T, act, lde, ldg, col_e, dim_pad};
  if (dtype == GL3_BF16 && mfma && d % 8 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)w % 16 == 0) {
    const unsigned tiles = (unsigned)((T + 15) / 16);
    if (T <= 256)
      side_gate_mfma_kernel<1, 16><<<dim3(tiles, (dim_pad + 15) / 16), dim3(1024), 0, stream>>>(x, (const bf16_t*)w, (const bf16_t*)table,
                                                                                               ids, (bf16_t*)g, s);
    else
      side_gate_mfma_kernel<2, 8><<<dim3(tiles, (dim_pad + 31) / 32), dim3(512), 0, stream>>>(x, (const bf16_t*)w, (const bf16_t*)table,
                                                                                             ids, (bf16_t*)g, s);
  } else {
    const dim3 grid(T, (dim_pad + 3) / 4), block(256);
    if (dtype == GL3_F32) side_gate_kernel<float><<<grid, block, 0, stream>>>(x, (const float*)w, (const float*)table, ids, (float*)g, s);
    else if (dtype == GL3_BF16) side_gate_kernel<bf16_t><<<grid, block, 0, stream>>>(x, (const bf16_t*)w, (const bf16_t*)table, ids, (bf16_t*)g, s);
    else GL3_REQUIRE(false, "gl3_side_gate: unknown dtype %d", dtype);
  }
  GL3_LAUNCH_CHECK();
  return 0;
}

// ----------------------------------------------------------------- x += y / rms(y) * w, and the norm after it
// One block a row, up to PER groups of 4 elements a thread, which stay in registers from the first read to the last
// write. With next_w: h [T][d] = row / sqrt(mean(row^2) + next_eps) * next_w in the type TH, and/or (xg not null, at most
// 64 rows) what a product that takes the norm over reads: xg = bfloat16(next_w * row), ssq[t] = the row's sum of squares.
template <int PER, typename TH>
__global__ __launch_bounds__(1024) void norm_add_next_kernel(float* __restrict__ x, const float* __restrict__ y,
                                                             const float* __restrict__ w, float eps, int d,
                                                             const float* __restrict__ next_w, float next_eps, TH* __restrict__ h,
                                                             bf16_t* __restrict__ xg, float* __restrict__ ssq) {
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  const int n4 = d / 4;
  ts_f32x4 v[PER];
  float s = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int i = threadIdx.x + p * blockDim.x;
    v[p] = i < n4 ? reinterpret_cast<const ts_f32x4*>(y + t * d)[i] : ts_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) s = fmaf(v[p][e], v[p][e], s);
  }
  const float inv = 1.0f / sqrtf(block_sum(s, scratch) / (float)d + eps);
  float ss = 0.f;
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int i = threadIdx.x + p * blockDim.x;
    if (i < n4) {
      ts_f32x4 row = reinterpret_cast<const ts_f32x4*>(x + t * d)[i];
      const ts_f32x4 wi = reinterpret_cast<const ts_f32x4*>(w)[i];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        row[e] += v[p][e] * inv * wi[e];
        ss = fmaf(row[e], row[e], ss);
      }
      reinterpret_cast<ts_f32x4*>(x + t * d)[i] = row;
      v[p] = row;
    }
  }
  if (!next_w) return;
  ss = block_sum(ss, scratch);
  if (ssq && threadIdx.x == 0) ssq[t] = ss;
  const float f = 1.0f / sqrtf(ss / (float)d + next_eps);
#pragma unroll
  for (int p = 0; p < PER; ++p) {
    const int i = threadIdx.x + p * blockDim.x;
    if (i >= n4) continue;
    const ts_f32x4 wi = reinterpret_cast<const ts_f32x4*>(next_w)[i];
    if (h) {
      typedef TH vec4 __attribute__((ext_vector_type(4)));
      vec4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = from_f32<TH>(v[p][e] * f * wi[e]);
      reinterpret_cast<vec4*>(h + t * d)[i] = o;
    }
    if (xg) {
      typedef bf16_t bvec4 __attribute__((ext_vector_type(4)));
      bvec4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = static_cast<bf16_t>(wi[e] * v[p][e]);
      reinterpret_cast<bvec4*>(xg + t * d)[i] = o;
    }
  }
}

extern "C" int gl3_norm_add_next(float* x, const float* y, const float* w, float eps, int T, int d, const float* next_w,
                                 float next_eps, void* h, int h_dtype, void* xg, float* ssq, hipStream_t stream) {
  if (T == 0) return 0;
  GL3_REQUIRE(x && y && w && T > 0 && d > 0 && d % 4 == 0 && d <= 32768, "gl3_norm_add_next: rows of %d", d);
  GL3_REQUIRE((uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)next_w % 16 == 0 &&
                  (uintptr_t)h % 16 == 0 && (uintptr_t)xg % 16 == 0, "gl3_norm_add_next: rows must be aligned to 16 bytes");
  GL3_REQUIRE((!h && !xg) || next_w, "gl3_norm_add_next: the next norm's rows without its weight");
  GL3_REQUIRE((xg == nullptr) == (ssq == nullptr) && (!ssq || T <= 64), "gl3_norm_add_next: sums of squares of %d rows", T);
  const int n4 = d / 4, threads = n4 >= 1024 ? 1024 : (n4 + 63) / 64 * 64, per = (n4 + threads - 1) / threads;
#define NA_GO(PER, TH) \
  norm_add_next_kernel<PER, TH><<<dim3(T), dim3(threads), 0, stream>>>(x, y, w, eps, d, next_w, next_eps, (TH*)h, (bf16_t*)xg, ssq)
#define NA_PER(TH)               \
  do {                           \
    if (per <= 1) NA_GO(1, TH);  \
    else if (per <= 2) NA_GO(2, TH); \
    else NA_GO(8, TH);           \
  } while (0)
  if (!h || h_dtype == GL3_BF16) NA_PER(bf16_t);
  else if (h_dtype == GL3_F32) NA_PER(float);
  else GL3_REQUIRE(false, "gl3_norm_add_next: unknown dtype %d", h_dtype);
#undef NA_PER
#undef NA_GO
  GL3_LAUNCH_CHECK();
  return 0;
}
