// Queries, keys and values behind a short causal convolution over time, turned, brought to unit root mean square and put
// where an attention reads them: one kernel from the rows of the stacked projection to the queries' rows and the cache.
//
// rows [T][ld]: a token's projected heads, queries (Hq heads of hs elements), keys (Kh of hs), values (Kh of vd), head
// sizes padded to multiples of 16 with zeros; C = (Hq + Kh) hs + Kh vd channels from column 0 on. Per channel
//   y[t] = w[taps - 1] u[t] + w[taps - 2] u[t - 1] + ...,   as far back as the sequence reaches,
// w [taps][C] float (the last row is the current token's). The inputs before a step's first token are what the sequence's
// slot holds: `held` [taps - 1][C] floats, oldest first, from `held_off` of the slot's state.
// Queries and keys: the pairs (2i, 2i + 1) of a head's first `rot` elements are turned by the token's position (tables
// [position][rot / 2]; null: no rotation), then the head is divided by sqrt(mean(x^2) + eps) over its `norm_dim` stored
// elements (eps < 0: no such norm) and multiplied by qw / kw (null: no weight). Queries go to q_out [T][Hq hs], keys and
// values to their places in the paged cache. All arithmetic is 32-bit.
#include "common.h"

struct ConvHeads {
  int Hq, Kh, hs, vd, taps, rot, norm_dim;
  long ld, state_stride, held_off;
  float eps;
  int table_stride, page_size, n_tokens, one_each;
};

template <typename T>
__device__ __forceinline__ void load8(const T* __restrict__ p, float (&out)[8]) {
  typedef T vec __attribute__((ext_vector_type(16 / sizeof(T))));
  constexpr int W = 16 / sizeof(T);
#pragma unroll
  for (int a = 0; a < 8 / W; ++a) {
    const vec x = *reinterpret_cast<const vec*>(p + a * W);
#pragma unroll
    for (int e = 0; e < W; ++e) out[a * W + e] = to_f32<T>(x[e]);
  }
}
template <typename T>
__device__ __forceinline__ void store8(T* __restrict__ p, const float (&in)[8]) {
  typedef T vec __attribute__((ext_vector_type(16 / sizeof(T))));
  constexpr int W = 16 / sizeof(T);
#pragma unroll
  for (int a = 0; a < 8 / W; ++a) {
    vec x;
#pragma unroll
    for (int e = 0; e < W; ++e) x[e] = from_f32<T>(in[a * W + e]);
    *reinterpret_cast<vec*>(p + a * W) = x;
  }
}

// The sums of the 8 channels from c on for token t of a sequence whose first token of this step is `first`. TAPS: the taps,
// 0 where only the launch knows them. The usual cases ask for everything at once, without a condition in between: a token
// whose whole reach lies in this step, and a sequence's first token of the step, whose earlier inputs the slot holds (with
// `move` these then move on: the sequence brings this one token, and nobody else reads these channels).
template <typename T, int TAPS>
__device__ __forceinline__ void conv8(const T* __restrict__ rows, const float* __restrict__ w, float* __restrict__ held,
                                      const ConvHeads& s, int C, int c, int t, int first, bool move, float (&y)[8]) {
  const int taps = TAPS ? TAPS : s.taps;
  constexpr int N = TAPS ? TAPS : 1;
#pragma unroll
  for (int e = 0; e < 8; ++e) y[e] = 0.f;
  if (TAPS && t - first >= taps - 1) {
    float u[N][8], f[N][8];
#pragma unroll
    for (int j = 0; j < N; ++j) {
      load8<T>(rows + (long)(t - (N - 1) + j) * s.ld + c, u[j]);
      load8<float>(w + (long)j * C + c, f[j]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) y[e] = fmaf(f[j][e], u[j][e], y[e]);
    return;
  }
  if (TAPS && t == first) {
    float u[N][8], f[N][8];
#pragma unroll
    for (int j = 0; j < N; ++j) {
      if (j + 1 < N) load8<float>(held + (long)j * C + c, u[j]);
      else load8<T>(rows + (long)t * s.ld + c, u[j]);
      load8<float>(w + (long)j * C + c, f[j]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) y[e] = fmaf(f[j][e], u[j][e], y[e]);
    if (move) {
#pragma unroll
      for (int j = 1; j < N; ++j) store8<float>(held + (long)(j - 1) * C + c, u[j]);
    }
    return;
  }
  for (int j = 0; j < taps; ++j) {
    const int src = t - (taps - 1) + j;
    float u[8], f[8];
    if (src >= first) load8<T>(rows + (long)src * s.ld + c, u);
    else load8<float>(held + (long)(src - first + taps - 1) * C + c, u);
    load8<float>(w + (long)j * C + c, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = fmaf(f[e], u[e], y[e]);
  }
  if (move) {
    float u[8];
    for (int j = 0; j + 2 < taps; ++j) {
      load8<float>(held + (long)(j + 1) * C + c, u);
      store8<float>(held + (long)j * C + c, u);
    }
    if (taps > 1) {
      load8<T>(rows + (long)t * s.ld + c, u);
      store8<float>(held + (long)(taps - 2) * C + c, u);
    }
  }
}

// A block a token (an XCD a stretch of tokens), or in a step of few tokens several: grid y, of which the last makes the
// values and the others the queries and keys. A query or key head takes `lp` lanes side by side, a power of two, 8
// channels each; the block whose token begins a group of 8 positions (or its sequence's tokens of this step) makes the
// values of the whole group, which lie together in the cache.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_heads_kernel(
    const T* __restrict__ rows, const float* __restrict__ w, float* __restrict__ state, const int* __restrict__ cu_seqlens,
    const int* __restrict__ seq_of_token, const int* __restrict__ slot_ids, const int* __restrict__ positions,
    const int* __restrict__ table_rows, const int* __restrict__ block_table, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, const float* __restrict__ qw, const float* __restrict__ kw, T* __restrict__ q_out,
    T* __restrict__ k_cache, T* __restrict__ v_cache, ConvHeads s, int lp) {
  const int per_xcd = (s.n_tokens + 7) / 8;
  const int t = ((int)blockIdx.x % 8) * per_xcd + (int)blockIdx.x / 8;
  if (t >= s.n_tokens) return;
  const int b = seq_of_token[t], first = cu_seqlens[b], last = cu_seqlens[b + 1];
  const int pos = positions[t];
  const long page = block_table[(long)table_rows[t] * s.table_stride + pos / s.page_size];
  const int in_page = pos % s.page_size;
  const int QK = (s.Hq + s.Kh) * s.hs, C = QK + s.Kh * s.vd, half = s.rot / 2;
  float* held = state + (long)slot_ids[b] * s.state_stride + s.held_off;
  const int heads = s.Hq + s.Kh, lanes = heads * lp;
  const int parts = gridDim.y, qk_parts = parts > 1 ? parts - 1 : 1;
  if ((int)blockIdx.y < qk_parts) {
    for (int i0 = 256 * blockIdx.y; i0 < lanes; i0 += 256 * qk_parts) {      // (whole waves: the sum over a head's lanes is theirs together)
      const int i = i0 + threadIdx.x, head = i / lp, e0 = (i % lp) * 8;
      const bool here = i < lanes && e0 < s.hs;
      const int c = here ? head * s.hs + e0 : 0;
      float y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (here) conv8<T, TAPS>(rows, w, held, s, C, c, t, first, s.one_each, y);
      if (cos_t && here && e0 < s.rot) {
#pragma unroll
        for (int a = 0; a < 4; ++a) {
          const int p = e0 / 2 + a;
          if (p < half) {
            const float cs = cos_t[(long)pos * half + p], sn = sin_t[(long)pos * half + p];
            const float u = y[2 * a], v = y[2 * a + 1];
            y[2 * a] = u * cs - v * sn;
            y[2 * a + 1] = v * cs + u * sn;
          }
        }
      }
      if (s.eps >= 0.f) {
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf(y[e], y[e], ss);
        for (int o = 1; o < lp; o <<= 1) ss += __shfl_xor(ss, o, 64);
        const float inv = 1.0f / sqrtf(ss / (float)s.norm_dim + s.eps);
        const float* nw = head < s.Hq ? qw : kw;
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] *= nw && here ? inv * nw[e0 + e] : inv;
      }
      if (here) {
        if (head < s.Hq) store8<T>(q_out + (long)t * s.Hq * s.hs + c, y);
        else store8<T>(k_cache + (page * s.Kh + head - s.Hq) * (long)s.page_size * s.hs + gl3_k_offset(in_page, e0, s.hs), y);
      }
    }
    if (parts > 1) return;
  }
  int run = 0;                                             // how many tokens' values this block makes
  if ((pos & 7) == 0 || t == first) {
    run = 8 - (pos & 7);
    if (run > last - t) run = last - t;
  }
  if (!run) return;
  const int per_head = s.vd / 8;
  for (int i = threadIdx.x; i < s.Kh * per_head; i += 256) {
    const int kvh = i / per_head, e0 = (i % per_head) * 8, c = QK + kvh * s.vd + e0;
    T* at = v_cache + (page * s.Kh + kvh) * (long)s.page_size * s.vd + gl3_v_offset(e0, in_page, s.page_size);
    if (run == 8) {                                        // (pos is a multiple of 8: 8 positions of a dimension lie together)
      T all[8][8];
#pragma unroll
      for (int r = 0; r < 8; ++r) {
        float y[8];
        conv8<T, TAPS>(rows, w, held, s, C, c, t + r, first, false, y);
#pragma unroll
        for (int e = 0; e < 8; ++e) all[e][r] = from_f32<T>(y[e]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        float o[8];
#pragma unroll
        for (int r = 0; r < 8; ++r) o[r] = to_f32<T>(all[e][r]);
        store8<T>(at + 8 * e, o);
      }
    } else {
      for (int r = 0; r < run; ++r) {                      // (one_each: run is 1)
        float y[8];
        conv8<T, TAPS>(rows, w, held, s, C, c, t + r, first, s.one_each, y);
#pragma unroll
        for (int e = 0; e < 8; ++e) at[8 * e + r] = from_f32<T>(y[e]);
      }
    }
  }
}

// grid (B, ceil(C / 256)): a thread moves one channel's held inputs on by its sequence's new tokens, oldest first, so that
// no place is written before it has been read.
template <typename T>
__global__ __launch_bounds__(256) void conv_heads_state_kernel(const T* __restrict__ rows, float* __restrict__ state,
                                                               const int* __restrict__ cu_seqlens,
                                                               const int* __restrict__ slot_ids, ConvHeads s, int C) {
  const int b = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int first = cu_seqlens[b], n = cu_seqlens[b + 1] - first;
  if (n <= 0) return;
  float* held = state + (long)slot_ids[b] * s.state_stride + s.held_off + c;
  for (int j = 0; j < s.taps - 1; ++j) {
    const int src = n - (s.taps - 1) + j;
    held[(long)j * C] = src >= 0 ? to_f32<T>(rows[(long)(first + src) * s.ld + c]) : held[(long)(j + n) * C];
  }
}

extern "C" int gl3_conv_heads(const void* rows, int dtype, long ld, const float* w, int taps, float* state, long state_stride,
                              long held_off, const int* cu_seqlens, const int* seq_of_token, const int* slot_ids,
                              const int* positions, const int* table_rows, const int* block_table, int table_stride,
                              const float* cos_t, const float* sin_t, int rot, const float* qw, const float* kw, int norm_dim,
                              float eps, void* q_out, void* k_cache, void* v_cache, int n_tokens, int n_seqs, int Hq, int Kh,
                              int hs, int vd, int page_size, int one_each, hipStream_t stream) {
  if (n_tokens == 0 || n_seqs == 0) return 0;
  GL3_REQUIRE(rows && w && state && cu_seqlens && seq_of_token && slot_ids && positions && table_rows && block_table && q_out &&
                  k_cache && v_cache && n_tokens > 0 && n_seqs > 0 && table_stride > 0, "gl3_conv_heads: bad arguments");
  GL3_REQUIRE(Hq > 0 && Kh > 0 && hs > 0 && hs % 16 == 0 && hs <= 512 && vd > 0 && vd % 16 == 0 && taps >= 1 && taps <= 64,
              "gl3_conv_heads: %d heads over %d of %d and %d elements, %d taps", Hq, Kh, hs, vd, taps);
  GL3_REQUIRE((cos_t == nullptr) == (sin_t == nullptr) && (!cos_t || (rot > 0 && rot % 2 == 0 && rot <= hs)),
              "gl3_conv_heads: %d rotated elements of %d", rot, hs);
  GL3_REQUIRE(eps < 0.f || (norm_dim > 0 && norm_dim <= hs), "gl3_conv_heads: a norm over %d of %d elements", norm_dim, hs);
  GL3_REQUIRE(page_size > 0 && page_size % 32 == 0, "gl3_conv_heads: pages of %d positions", page_size);
  const long C = (long)(Hq + Kh) * hs + (long)Kh * vd;
  GL3_REQUIRE(C <= ld && ld % 8 == 0 && C < (1L << 30) && held_off >= 0 && held_off + C * (taps - 1) <= state_stride,
              "gl3_conv_heads: %ld channels in rows of %ld, a slot's state of %ld floats from %ld", C, ld, state_stride, held_off);
  GL3_REQUIRE((uintptr_t)rows % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)q_out % 16 == 0 && (uintptr_t)k_cache % 16 == 0 &&
                  (uintptr_t)v_cache % 16 == 0 && (uintptr_t)state % 16 == 0 && state_stride % 4 == 0 && held_off % 4 == 0,
              "gl3_conv_heads: rows, weights, state and cache must be aligned to 16 bytes");
  GL3_REQUIRE(!one_each || n_tokens == n_seqs, "gl3_conv_heads: %d tokens of %d sequences are not one each", n_tokens, n_seqs);
  int lp = 1;
  while (lp * 8 < hs) lp *= 2;
  const ConvHeads s{Hq, Kh, hs, vd, taps, cos_t ? rot : 0, norm_dim, ld, state_stride, held_off, eps, table_stride, page_size,
                    n_tokens, one_each};
  const unsigned parts = n_tokens <= 64 ? (unsigned)(((Hq + Kh) * lp + 255) / 256 + 1) : 1;
  const dim3 grid((unsigned)((n_tokens + 7) / 8 * 8), parts), block(256), sgrid(n_seqs, (unsigned)((C + 255) / 256));
#define CH_TAPS(T, TAPS)                                                                                                     \
  conv_heads_kernel<T, TAPS><<<grid, block, 0, stream>>>((const T*)rows, w, state, cu_seqlens, seq_of_token, slot_ids,       \
                                                         positions, table_rows, block_table, cos_t, sin_t, qw, kw, (T*)q_out, \
                                                         (T*)k_cache, (T*)v_cache, s, lp)
#define CH_GO(T)                                                                                                              \
  do {                                                                                                                        \
    if (taps == 2) CH_TAPS(T, 2);                                                                                             \
    else if (taps == 3) CH_TAPS(T, 3);                                                                                        \
    else if (taps == 4) CH_TAPS(T, 4);                                                                                        \
    else CH_TAPS(T, 0);                                                                                                       \
    if (taps > 1 && !one_each) {                                                                                              \
      GL3_LAUNCH_CHECK();                                                                                                     \
      conv_heads_state_kernel<T><<<sgrid, block, 0, stream>>>((const T*)rows, state, cu_seqlens, slot_ids, s, (int)C);        \
    }                                                                                                                         \
  } while (0)
  if (dtype == GL3_F32) CH_GO(float);
  else if (dtype == GL3_BF16) CH_GO(bf16_t);
  else GL3_REQUIRE(false, "gl3_conv_heads: unknown dtype %d", dtype);
#undef CH_GO
#undef CH_TAPS
  GL3_LAUNCH_CHECK();
  return 0;
}
