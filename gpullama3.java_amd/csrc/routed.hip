// A mixture of experts: the choice of a token's experts, the rows of (token, choice) pairs ordered by expert, the
// experts' products over those rows, and the weighted sum per token.
//
// A pair's result depends on its token and its expert alone: the order of the pairs inside an expert's run and the
// tile a pair falls into change nothing, so a token's output does not depend on its batch-mates. Sums over K run in an
// order that the shapes fix.
#include "common.h"

#define ROUTE_MAX_TOP 16
#define ROUTE_MAX_EXPERTS 1024

// ----------------------------------------------------------------- the choice
// logits [T][E] float. The `top` largest (the lower number wins a tie) -> idx [T][top]; their weights are the softmax
// over the chosen logits alone -> wts [T][top]. One thread a token.
// With `scores` set the rule is another: s = softmax over all E logits; the choice goes by s + correction[e]
// (correction may be null), the weights are the chosen s themselves divided by their sum plus sum_eps.
// A third rule (scores 2): s = sigmoid of every logit, the largest are chosen, their weights are their s as they are.
//
// RouteExtras: rows of logits of `ld` floats. `in_wts` (not null): a pair's weight multiplies its expert's INPUT: it is
// written here and the weight of its output (wts) is 1. `gate_col` (not negative): the output of the expert that
// every token passes is multiplied by sigmoid(logits[gate_col]), which goes to that expert's pair in wts, or to gate_out
// [T] where it has no pair. ssq (not null): the rows that the experts will multiply are not normed yet; [n_partials][64]
// partial sums of squares of the residual rows (at most 64 of them), from which 1 / sqrt(sum / d + eps) is made and
// multiplied into in_wts (for a pair whose weight is 1 too) and handed out as norm_out [T].
// n_groups > 1 (rule 1): of every E / n_groups experts in a row the best one speaks for all; the `keep` groups whose speakers
// stand first stay open, the others' experts are out of the choice (the lower number wins a tie). weight_scale
// multiplies the chosen experts' weights.
struct RouteExtras {
  int ld;
  float* in_wts;
  int gate_col;
  float* gate_out;
  const float* ssq;
  int n_partials, d;
  float eps;
  float* norm_out;
  int n_groups, keep;
  float weight_scale;
};

// Rule 1 by a whole wave: lane l works for the experts l, l + 64, ... c: this wave's share of shared memory, E scores, n_groups
// group scores, and ROUTE_MAX_TOP chosen scores and numbers. Nothing is passed from lane to lane: every lane reads what the
// others wrote. Up to 256 experts are chosen by rank (a lane counts the experts in front of its own), more by one search for
// the largest after the other.
__device__ __forceinline__ void wave_argmax(float& v, int& i) {      // the largest v, of equal ones the lowest i
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o, 64);
    const int oi = __shfl_xor(i, o, 64);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}
__device__ __forceinline__ void wave_lds_order() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
// how many of the n values stand in front of value v with number i
__device__ __forceinline__ int rank_among(const float* c, int n, float v, int i) {
  int r = 0;
#pragma unroll 4
  for (int e = 0; e < n; ++e) r += c[e] > v || (c[e] == v && e < i);
  return r;
}
#define ROUTE_BY_RANK 256
#define ROUTE_WAVE_FLOATS(E, groups) ((E) + (groups) + 2 * ROUTE_MAX_TOP)
__device__ __forceinline__ void route_choose_scores(const float* __restrict__ logits, int t, int E, int top, int* idx,
                                                    float* __restrict__ wts, int always, const float* __restrict__ correction,
                                                    float sum_eps, const RouteExtras& x, float inv_rms, float* c) {
  const float* z = logits + (long)t * x.ld;
  const int lane = threadIdx.x & 63, stride = top + (always >= 0 ? 1 : 0), per = E / x.n_groups;
  float* gs = c + E;
  float* chosen_s = gs + x.n_groups;
  int* chosen_e = reinterpret_cast<int*>(chosen_s + ROUTE_MAX_TOP);
  const bool by_rank = E <= ROUTE_BY_RANK;
  float s[ROUTE_BY_RANK / 64];             // the scores of this lane's experts, where they are few
  wave_lds_order();                        // (the wave's last token is done with its share)
  if (lane < top) {                        // (no number among the scores: any experts, but some that exist)
    chosen_s[lane] = 0.f;
    chosen_e[lane] = lane;
  }
  float z_max = -INFINITY, z_sum = 0.f;
  for (int e = lane; e < E; e += 64) c[e] = z[e];
  wave_lds_order();
  if (by_rank) {
#pragma unroll 4
    for (int e = 0; e < E; ++e) z_max = fmaxf(z_max, c[e]);
    wave_lds_order();
#pragma unroll
    for (int n = 0; n < ROUTE_BY_RANK / 64; ++n)
      if (lane + 64 * n < E) c[lane + 64 * n] = s[n] = expf(c[lane + 64 * n] - z_max);
    wave_lds_order();
#pragma unroll 4
    for (int e = 0; e < E; ++e) z_sum += c[e];
    wave_lds_order();
#pragma unroll
    for (int n = 0; n < ROUTE_BY_RANK / 64; ++n)
      if (lane + 64 * n < E) {
        s[n] /= z_sum;
        c[lane + 64 * n] = s[n] + (correction ? correction[lane + 64 * n] : 0.f);
      }
  } else {
    for (int e = lane; e < E; e += 64) z_max = fmaxf(z_max, c[e]);
    z_max = wave_max(z_max);
    for (int e = lane; e < E; e += 64) z_sum += expf(c[e] - z_max);
    z_sum = wave_sum(z_sum);
    for (int e = lane; e < E; e += 64) c[e] = expf(c[e] - z_max) / z_sum + (correction ? correction[e] : 0.f);
  }
  wave_lds_order();
  if (x.n_groups > 1) {
    for (int g = lane; g < x.n_groups; g += 64) {
      float m = -INFINITY;
      for (int i = 0; i < per; ++i) m = fmaxf(m, c[g * per + i]);
      gs[g] = m;
    }
    wave_lds_order();
    for (int g = lane; g < x.n_groups; g += 64)
      if (rank_among(gs, x.n_groups, gs[g], g) >= x.keep)
        for (int i = 0; i < per; ++i) c[g * per + i] = -INFINITY;
    wave_lds_order();
  }
  if (by_rank) {
#pragma unroll
    for (int n = 0; n < ROUTE_BY_RANK / 64; ++n) {
      const int e = lane + 64 * n;
      if (e < E && c[e] > -INFINITY) {
        const int rank = rank_among(c, E, c[e], e);
        if (rank < top) {
          chosen_s[rank] = s[n];
          chosen_e[rank] = e;
        }
      }
    }
  } else {
    for (int j = 0; j < top; ++j) {
      float v = -INFINITY;
      int best = 0x7fffffff;
      for (int e = lane; e < E; e += 64)
        if (c[e] > v) {
          v = c[e];
          best = e;
        }
      wave_argmax(v, best);
      if (best < E && (best & 63) == lane) {
        chosen_s[j] = expf(z[best] - z_max) / z_sum;
        chosen_e[j] = best;
        c[best] = -INFINITY;
      }
    }
  }
  wave_lds_order();
  float sum = 0.f;
  for (int j = 0; j < top; ++j) sum += chosen_s[j];
  sum += sum_eps;
  if (lane < top) {
    const float w = chosen_s[lane] / sum * x.weight_scale;
    idx[(long)t * stride + lane] = chosen_e[lane];
    wts[(long)t * stride + lane] = x.in_wts ? 1.0f : w;
    if (x.in_wts) x.in_wts[(long)t * stride + lane] = w * inv_rms;
  }
  if (lane == 0) {
    const float gate = x.gate_col >= 0 ? 1.0f / (1.0f + expf(-z[x.gate_col])) : 1.0f;
    if (always >= 0) {
      idx[(long)t * stride + top] = always;
      wts[(long)t * stride + top] = gate;
      if (x.in_wts) x.in_wts[(long)t * stride + top] = inv_rms;
    }
    if (x.gate_out) x.gate_out[t] = gate;
    if (x.norm_out) x.norm_out[t] = inv_rms;
  }
}

// Rules 0 and 2, a thread a token.
__device__ __forceinline__ void route_choose(const float* __restrict__ logits, int t, int E, int top, int* idx,
                                             float* __restrict__ wts, int always, int scores, const RouteExtras& x,
                                             float inv_rms) {
  const float* z = logits + (long)t * x.ld;
  const int stride = top + (always >= 0 ? 1 : 0);
  int chosen[ROUTE_MAX_TOP];
  float val[ROUTE_MAX_TOP];
  for (int j = 0; j < top; ++j) {
    int best = -1;
    float bv = -INFINITY;
    for (int e = 0; e < E; ++e) {
      bool taken = false;
      for (int i = 0; i < j; ++i) taken |= chosen[i] == e;
      if (!taken && (best < 0 || z[e] > bv)) {      // (a sigmoid keeps the logits' order)
        best = e;
        bv = z[e];
      }
    }
    chosen[j] = best;
    val[j] = bv;
  }
  float sum = 0.f;
  if (scores == 2) {
    for (int j = 0; j < top; ++j) val[j] = 1.0f / (1.0f + expf(-val[j]));
    sum = 1.f;
  } else {
    const float largest = val[0];          // (the first chosen is the largest)
    for (int j = 0; j < top; ++j) {
      val[j] = expf(val[j] - largest);
      sum += val[j];
    }
  }
  for (int j = 0; j < top; ++j) {
    idx[(long)t * stride + j] = chosen[j];
    const float w = val[j] / sum * x.weight_scale;
    wts[(long)t * stride + j] = x.in_wts ? 1.0f : w;
    if (x.in_wts) x.in_wts[(long)t * stride + j] = w * inv_rms;
  }
  const float gate = x.gate_col >= 0 ? 1.0f / (1.0f + expf(-z[x.gate_col])) : 1.0f;
  if (always >= 0) {                     // one more pair per token: the expert that every token passes, with weight 1
    idx[(long)t * stride + top] = always;
    wts[(long)t * stride + top] = gate;
    if (x.in_wts) x.in_wts[(long)t * stride + top] = inv_rms;
  }
  if (x.gate_out) x.gate_out[t] = gate;
  if (x.norm_out) x.norm_out[t] = inv_rms;
}

__global__ __launch_bounds__(64) void route_topk_kernel(const float* __restrict__ logits, int T, int E, int top,
                                                         int* __restrict__ idx, float* __restrict__ wts, int always, int scores,
                                                         RouteExtras x) {
  const int t = blockIdx.x * 64 + threadIdx.x;
  if (t < T) route_choose(logits, t, E, top, idx, wts, always, scores, x, 1.0f);
}

// rule 1: a wave a token, four a block
__global__ __launch_bounds__(256) void route_scores_kernel(const float* __restrict__ logits, int T, int E, int top,
                                                           int* __restrict__ idx, float* __restrict__ wts, int always,
                                                           const float* __restrict__ correction, float sum_eps, RouteExtras x) {
  extern __shared__ float route_lds[];      // ROUTE_WAVE_FLOATS a wave
  const int wave = threadIdx.x >> 6, t = blockIdx.x * 4 + wave;
  if (t < T)
    route_choose_scores(logits, t, E, top, idx, wts, always, correction, sum_eps, x, 1.0f, route_lds + wave * ROUTE_WAVE_FLOATS(E, x.n_groups));
}

// ----------------------------------------------------------------- pairs ordered by expert
// idx [n_pairs] -> offsets [E + 1] (the first place of each expert's run) and sorted [n_pairs] (the pairs, expert by
// expert). One block.
__device__ __forceinline__ void route_order(const int* idx, int n_pairs, int E, int* __restrict__ offsets,
                                            int* __restrict__ sorted) {
  __shared__ int count[ROUTE_MAX_EXPERTS + 1];
  __shared__ int cursor[ROUTE_MAX_EXPERTS];
  for (int e = threadIdx.x; e <= E; e += blockDim.x) count[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n_pairs; i += blockDim.x) atomicAdd(&count[idx[i]], 1);
  __syncthreads();
  if (threadIdx.x == 0) {
    int run = 0;
    for (int e = 0; e < E; ++e) {
      const int c = count[e];
      count[e] = run;
      cursor[e] = run;
      run += c;
    }
    count[E] = run;
  }
  __syncthreads();
  for (int e = threadIdx.x; e <= E; e += blockDim.x) offsets[e] = count[e];
  for (int i = threadIdx.x; i < n_pairs; i += blockDim.x) sorted[atomicAdd(&cursor[idx[i]], 1)] = i;
}

__global__ __launch_bounds__(1024) void route_sort_kernel(const int* __restrict__ idx, int n_pairs, int E,
                                                           int* __restrict__ offsets, int* __restrict__ sorted) {
  route_order(idx, n_pairs, E, offsets, sorted);
}

// Both in one launch for a step of at most 1024 tokens (a thread a token, then the block orders the pairs).
__global__ __launch_bounds__(1024) void route_few_kernel(const float* __restrict__ logits, int T, int E, int top,
                                                          int* idx, float* __restrict__ wts,
                                                          int* __restrict__ offsets, int* __restrict__ sorted, int always,
                                                          int scores, const float* __restrict__ correction, float sum_eps,
                                                          RouteExtras x, int choosers) {
  extern __shared__ float route_lds[];      // rule 1: ROUTE_WAVE_FLOATS for each of the `choosers` waves
  __shared__ float inv_rms[64];
  if (x.ssq) {                              // (the same for all threads) a wave a row adds up its partial sums
    for (int t = threadIdx.x >> 6; t < T; t += blockDim.x >> 6) {
      float s = 0.f;
      for (int i = threadIdx.x & 63; i < x.n_partials; i += 64) s += x.ssq[(long)i * 64 + t];
      s = wave_sum(s);
      if ((threadIdx.x & 63) == 0) inv_rms[t] = 1.0f / sqrtf(s / (float)x.d + x.eps);
    }
    __syncthreads();
  }
  if (scores == 1) {
    const int wave = threadIdx.x >> 6;
    if (wave < choosers)
      for (int t = wave; t < T; t += choosers)
        route_choose_scores(logits, t, E, top, idx, wts, always, correction, sum_eps, x, x.ssq ? inv_rms[t] : 1.0f,
                            route_lds + wave * ROUTE_WAVE_FLOATS(E, x.n_groups));
  } else if ((int)threadIdx.x < T) {
    route_choose(logits, threadIdx.x, E, top, idx, wts, always, scores, x, x.ssq ? inv_rms[threadIdx.x] : 1.0f);
  }
  __threadfence_block();
  __syncthreads();
  const int more = always >= 0 ? 1 : 0;
  route_order(idx, T * (top + more), E + more, offsets, sorted);
}

// `always` (-1: none): the number E of one more expert behind the router's, which every token passes with weight 1; idx
// and wts then have top + 1 entries a token, offsets E + 2.
extern "C" int gl3_route(const float* logits, int n_tokens, int E, int top, int* idx, float* wts, int* offsets, int* sorted,
                         int always, int scores, const float* correction, float sum_eps, int ld, float* in_wts, int gate_col,
                         float* gate_out, const float* ssq, int n_partials, int d, float eps, float* norm_out, int n_groups,
                         int keep, float weight_scale, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  GL3_REQUIRE(logits && idx && wts && offsets && sorted, "gl3_route: null argument");
  const int more = always >= 0 ? 1 : 0;
  GL3_REQUIRE(n_tokens > 0 && E >= 1 && E + more <= ROUTE_MAX_EXPERTS && top >= 1 && top <= ROUTE_MAX_TOP && top <= E,
              "gl3_route: the %d largest of %d experts (at most %d of %d)", top, E, ROUTE_MAX_TOP, ROUTE_MAX_EXPERTS);
  GL3_REQUIRE(always < 0 || always == E, "gl3_route: the expert that every token passes is number %d, not %d", E, always);
  GL3_REQUIRE(scores >= 0 && scores <= 2 && ld >= E && gate_col < ld, "gl3_route: rule %d, rows of %d for %d experts, gate in column %d",
              scores, ld, E, gate_col);
  GL3_REQUIRE(!gate_out || gate_col >= 0, "gl3_route: a gate to hand out without a column of logits for it");
  GL3_REQUIRE(!ssq || (n_tokens <= 64 && n_partials > 0 && d > 0 && in_wts),
              "gl3_route: a norm carried by the pairs' weights takes at most 64 tokens and weights on the experts' inputs");
  GL3_REQUIRE(n_groups >= 1 && (n_groups == 1 || (scores == 1 && E % n_groups == 0 && keep >= 1 && keep <= n_groups &&
                                                  top <= keep * (E / n_groups))),
              "gl3_route: the %d largest of %d experts in the best %d of %d groups", top, E, keep, n_groups);
  const RouteExtras x{ld, in_wts, gate_col, gate_out, ssq, n_partials, d, eps, norm_out, n_groups, keep, weight_scale};
  const size_t per_wave = (size_t)ROUTE_WAVE_FLOATS(E, n_groups) * sizeof(float);
  if (n_tokens <= 64) {
    int choosers = (int)(40 * 1024 / per_wave);      // (beside the counters of the ordering)
    choosers = choosers > 16 ? 16 : choosers;
    route_few_kernel<<<dim3(1), dim3(1024), scores == 1 ? choosers * per_wave : 0, stream>>>(
        logits, n_tokens, E, top, idx, wts, offsets, sorted, always, scores, correction, sum_eps, x, choosers);
    GL3_LAUNCH_CHECK();
    return 0;
  }
  if (scores == 1)
    route_scores_kernel<<<dim3((n_tokens + 3) / 4), dim3(256), 4 * per_wave, stream>>>(logits, n_tokens, E, top, idx, wts, always,
                                                                                     correction, sum_eps, x);
  else
    route_topk_kernel<<<dim3((n_tokens + 63) / 64), dim3(64), 0, stream>>>(logits, n_tokens, E, top, idx, wts, always, scores, x);
  GL3_LAUNCH_CHECK();
  route_sort_kernel<<<dim3(1), dim3(1024), 0, stream>>>(idx, n_tokens * (top + more), E + more, offsets, sorted);
  GL3_LAUNCH_CHECK();
  return 0;
}

// ----------------------------------------------------------------- the experts' products
// out[pair][n] = act(sum_k A[pair / a_div][k] * W[e][n][k]) for every pair of expert e's run. offsets null: one expert
// over all n_rows rows in their own order (the expert that every token passes). Tiles of TM rows of a run x TN columns;
// a block finds its run by walking the offsets (at most n_rows / TM + E tiles exist; a block beyond them leaves).
__device__ __forceinline__ float gl3_expert_act(float v, int act) {
  if (act == 1) return 0.5f * v * (1.0f + erff(v * 0.70710678118654752f));        // gelu, the erf form
  if (act == 2) return gl3_activation<false>(v, GL3_ACT_GELU_TANH);
  if (act == 3) return gl3_activation<false>(v, GL3_ACT_SILU);
  return v;
}

// A gated expert: the rows of W are gate and up in turns (row 2 n the gate's, row 2 n + 1 the up's row n), so a lane that
// holds column c of the sums finds its partner's in the lane beside it; the even one writes column c / 2 of the
// output: act(gate) * (up + shift), both bounded by `limit` first where it is positive (gl3_gated). Every lane of a
// wave must come here (the partner's value travels from lane to lane); `ok` says whether this lane's element exists.
// RowFactors: numbers per row (pair) that may be null: `in` multiplies the row's input (its sums, in front of the
// activation), `out` its output (behind it).
struct RowFactors {
  const float* in;
  const float* out;
};
// (A kernel brings them into shared memory with its rows, before the products: at the end a row's number, then its
// factor, would be two more trips to memory.)
__device__ __forceinline__ void factors_here(const RowFactors& f, int row, float* in, float* out) {
  *in = f.in && row >= 0 ? f.in[row] : 1.f;
  *out = f.out && row >= 0 ? f.out[row] : 1.f;
}
template <typename TO>
__device__ __forceinline__ void expert_store(TO* __restrict__ out, long ldo, int row, int n, bool ok, float v, int act,
                                             int gate_act, float limit, float shift, float before, float after) {
  v *= before;
  if (gate_act < 0) {
    if (ok) out[(long)row * ldo + n] = from_f32<TO>(gl3_expert_act(v, act) * after);
    return;
  }
  const float up = __shfl_xor(v, 1, 64);
  if (ok && !(n & 1)) out[(long)row * ldo + (n >> 1)] = from_f32<TO>(gl3_gated<false>(v, up, gate_act, limit, shift) * after);
}

__device__ __forceinline__ bool expert_tile(const int* offsets, int E, int n_rows, int TM, int tile, int* e_out, int* lo_out,
                                            int* hi_out) {
  if (!offsets) {
    *e_out = 0;
    *lo_out = tile * TM;
    *hi_out = n_rows;
    return tile * TM < n_rows;
  }
  for (int e = 0; e < E; ++e) {
    const int lo = offsets[e], hi = offsets[e + 1];
    const int nt = (hi - lo + TM - 1) / TM;
    if (tile < nt) {
      *e_out = e;
      *lo_out = lo + tile * TM;
      *hi_out = hi;
      return true;
    }
    tile -= nt;
  }
  return false;
}

#define EG_TM 16
#define EG_TN 64
#define EG_TK 32
template <typename TA, typename TW, typename TO>
__global__ __launch_bounds__(256) void expert_gemm_generic_kernel(const TA* __restrict__ A, long lda, int a_div,
                                                                   const TW* __restrict__ W, int N, int K,
                                                                   const int* __restrict__ offsets,
                                                                   const int* __restrict__ sorted, int E, int n_rows,
                                                                   TO* __restrict__ out, long ldo, int act, int gate_act, float limit,
                                                                   float shift, RowFactors rf) {
  __shared__ float sa[EG_TM][EG_TK + 1];
  __shared__ float sw[EG_TN][EG_TK + 1];
  __shared__ int rows[EG_TM];
  __shared__ float f_in[EG_TM], f_out[EG_TM];
  int e, lo, hi;
  if (!expert_tile(offsets, E, n_rows, EG_TM, blockIdx.x, &e, &lo, &hi)) return;
  const int m = hi - lo < EG_TM ? hi - lo : EG_TM;
  if (threadIdx.x < EG_TM) {
    const int row = threadIdx.x < m ? (sorted ? sorted[lo + threadIdx.x] : lo + threadIdx.x) : -1;
    rows[threadIdx.x] = row;
    factors_here(rf, row, &f_in[threadIdx.x], &f_out[threadIdx.x]);
  }
  __syncthreads();
  const int n0 = blockIdx.y * EG_TN;
  const TW* We = W + (long)e * N * K;
  const int r = threadIdx.x / 16, cg = threadIdx.x % 16;      // this thread: row r, columns cg + 16 j
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += EG_TK) {
    for (int i = threadIdx.x; i < EG_TM * EG_TK; i += 256) {
      const int rr = i / EG_TK, kk = i % EG_TK;
      sa[rr][kk] = (rows[rr] >= 0 && k0 + kk < K) ? to_f32<TA>(A[(long)(rows[rr] / a_div) * lda + k0 + kk]) : 0.f;
    }
    for (int i = threadIdx.x; i < EG_TN * EG_TK; i += 256) {
      const int nn = i / EG_TK, kk = i % EG_TK;
      sw[nn][kk] = (n0 + nn < N && k0 + kk < K) ? to_f32<TW>(We[(long)(n0 + nn) * K + k0 + kk]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < EG_TK; ++kk) {
      const float a = sa[r][kk];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = fmaf(a, sw[cg + 16 * j][kk], acc[j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = n0 + cg + 16 * j;
    expert_store<TO>(out, ldo, rows[r], n, rows[r] >= 0 && n < N, acc[j], act, gate_act, limit, shift,
                     f_in[r], f_out[r]);
  }
}

// The same on the matrix cores for bfloat16: a block of 4 waves works a tile of 64 rows x 64 columns, wave w the
// columns 16 w .. 16 w + 15 of all four row groups; operands come straight from memory, 4 consecutive k a lane (a
// row of A or of W per lane, as v_mfma_f32_16x16x16_bf16 takes them). K must be a multiple of 16.
typedef __attribute__((__vector_size__(4 * sizeof(short)))) short short4_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float float4_t;
#define EM_TM 64
#define EM_TN 64
template <typename TO>
__global__ __launch_bounds__(256) void expert_gemm_mfma_kernel(const bf16_t* __restrict__ A, long lda, int a_div,
                                                                const bf16_t* __restrict__ W, int N, int K,
                                                                const int* __restrict__ offsets,
                                                                const int* __restrict__ sorted, int E, int n_rows,
                                                                TO* __restrict__ out, long ldo, int act, int gate_act, float limit,
                                                                   float shift, RowFactors rf) {
  __shared__ int rows[EM_TM];
  __shared__ float f_in[EM_TM], f_out[EM_TM];
  int e, lo, hi;
  if (!expert_tile(offsets, E, n_rows, EM_TM, blockIdx.x, &e, &lo, &hi)) return;
  const int m = hi - lo < EM_TM ? hi - lo : EM_TM;
  if (threadIdx.x < EM_TM) {
    const int row = threadIdx.x < m ? (sorted ? sorted[lo + threadIdx.x] : lo + threadIdx.x) : -1;
    rows[threadIdx.x] = row;
    factors_here(rf, row, &f_in[threadIdx.x], &f_out[threadIdx.x]);
  }
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int li = lane & 15, kb = (lane >> 4) * 4;           // operand row / column of this lane, and its 4 k
  const int n = blockIdx.y * EM_TN + wave * 16 + li;
  const bf16_t* wp = W + ((long)e * N + (n < N ? n : 0)) * K + kb;
  const bf16_t* ap[4];
  bool a_ok[4];
#pragma unroll
  for (int g = 0; g < 4; ++g) {
    const int row = rows[g * 16 + li];
    a_ok[g] = row >= 0;
    ap[g] = A + (long)(row >= 0 ? row / a_div : 0) * lda + kb;
  }
  float4_t acc[4];
#pragma unroll
  for (int g = 0; g < 4; ++g) acc[g] = float4_t{0.f, 0.f, 0.f, 0.f};
  const int groups = (m + 15) / 16;
  for (int k0 = 0; k0 < K; k0 += 16) {
    short4_t b = {0, 0, 0, 0};
    if (n < N) b = *reinterpret_cast<const short4_t*>(wp + k0);
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      if (g < groups) {
        short4_t a = {0, 0, 0, 0};
        if (a_ok[g]) a = *reinterpret_cast<const short4_t*>(ap[g] + k0);
        acc[g] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(a, b, acc[g], 0, 0, 0);
      }
    }
  }
  // a lane holds column li of rows 4 (lane / 16) .. + 3 of every group
  const int nc = blockIdx.y * EM_TN + wave * 16 + li;
#pragma unroll
  for (int g = 0; g < 4; ++g) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = g * 16 + (lane >> 4) * 4 + i, row = rows[r];
      expert_store<TO>(out, ldo, row, nc, row >= 0 && nc < N, acc[g][i], act, gate_act, limit, shift, f_in[r], f_out[r]);
    }
  }
}

// For few rows (decode steps: an expert's run is a handful of pairs, and the time goes into reading its weights
// once): a block of 8 waves works a tile of 16 G rows of one run x 16 columns (G = 1, 2 or 4 by the runs' mean length,
// so that a run is mostly one tile and its weights are read once), wave w a slice of K (the slices follow from K
// alone), 32 k a step with v_mfma_f32_16x16x32_bf16: a lane holds 8 consecutive k of a row of A and of a row of W,
// read 16 bytes at a time, four steps in flight. The slices' sums are added in their order through shared memory.
typedef __bf16 bf16x8_few_t __attribute__((ext_vector_type(8)));
#define EF_WAVES 8
#define EF_TN 16
template <typename TO, int G>
__global__ __launch_bounds__(EF_WAVES * 64) void expert_gemm_few_kernel(const bf16_t* __restrict__ A, long lda, int a_div,
                                                                        const bf16_t* __restrict__ W, int N, int K,
                                                                        const int* __restrict__ offsets,
                                                                        const int* __restrict__ sorted, int E, int n_rows,
                                                                        TO* __restrict__ out, long ldo, int act, int gate_act, float limit,
                                                                   float shift, RowFactors rf) {
  constexpr int TM = 16 * G;
  __shared__ int rows[TM];
  __shared__ float f_in[TM], f_out[TM];
  __shared__ float part[EF_WAVES][TM][EF_TN + 1];
  int e, lo, hi;
  if (!expert_tile(offsets, E, n_rows, TM, blockIdx.x, &e, &lo, &hi)) return;
  const int m = hi - lo < TM ? hi - lo : TM;
  int my_row = -1;
  if (threadIdx.x < TM) {
    my_row = (int)threadIdx.x < m ? (sorted ? sorted[lo + threadIdx.x] : lo + threadIdx.x) : -1;
    rows[threadIdx.x] = my_row;
  }
  __syncthreads();
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int li = lane & 15, kg = (lane >> 4) * 8;
  const int n = blockIdx.y * EF_TN + li;
  const int per = ((K + 31) / 32 + EF_WAVES - 1) / EF_WAVES * 32;       // this wave's slice of K
  const int k_lo = wave * per, k_hi = k_lo + per < K ? k_lo + per : K;
  const int groups = (m + 15) / 16;
  const bf16_t* wp = W + ((long)e * N + (n < N ? n : N - 1)) * K + kg;
  const bf16_t* ap[G];
#pragma unroll
  for (int g = 0; g < G; ++g) {
    const int row = rows[g * 16 + li];                  // (rows beyond the run read the run's first row; their results are dropped)
    ap[g] = A + (long)((row >= 0 ? row : rows[0]) / a_div) * lda + kg;
  }
  float my_in = 1.f, my_out = 1.f;              // (asked for here, needed at the end)
  if (threadIdx.x < TM) factors_here(rf, my_row, &my_in, &my_out);
  const bf16x8_few_t zero = {0, 0, 0, 0, 0, 0, 0, 0};
  float4_t acc[G];
#pragma unroll
  for (int g = 0; g < G; ++g) acc[g] = float4_t{0.f, 0.f, 0.f, 0.f};
  int k0 = k_lo;
  for (; k0 + 128 <= k_hi; k0 += 128) {
    bf16x8_few_t a[4][G], b[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      b[u] = *reinterpret_cast<const bf16x8_few_t*>(wp + k0 + 32 * u);
#pragma unroll
      for (int g = 0; g < G; ++g)
        if (g < groups) a[u][g] = *reinterpret_cast<const bf16x8_few_t*>(ap[g] + k0 + 32 * u);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int g = 0; g < G; ++g)
        if (g < groups) acc[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u][g], b[u], acc[g], 0, 0, 0);
  }
  for (; k0 < k_hi; k0 += 32) {
    const bool in = k0 + kg < k_hi;                     // (K is a multiple of 8: a lane's 8 k lie inside or outside)
    const bf16x8_few_t b = in ? *reinterpret_cast<const bf16x8_few_t*>(wp + k0) : zero;
#pragma unroll
    for (int g = 0; g < G; ++g) {
      if (g < groups) {
        const bf16x8_few_t a = in ? *reinterpret_cast<const bf16x8_few_t*>(ap[g] + k0) : zero;
        acc[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[g], 0, 0, 0);
      }
    }
  }
  // a lane holds column li of rows 4 (lane / 16) .. + 3 of every group
  if (threadIdx.x < TM) {
    f_in[threadIdx.x] = my_in;
    f_out[threadIdx.x] = my_out;
  }
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][g * 16 + (lane >> 4) * 4 + i][li] = acc[g][i];
  __syncthreads();
  for (int base = 0; base < m * EF_TN; base += EF_WAVES * 64) {      // (every lane of a wave that has work walks along)
    const int idx = base + threadIdx.x;
    const bool in = idx < m * EF_TN;
    const int r = in ? idx / EF_TN : 0, c = idx % EF_TN;
    float sum = 0.f;
#pragma unroll
    for (int w = 0; w < EF_WAVES; ++w) sum += part[w][r][c];
    const int nc = blockIdx.y * EF_TN + c;
    expert_store<TO>(out, ldo, rows[r], nc, in && nc < N, sum, act, gate_act, limit, shift, f_in[r], f_out[r]);
  }
}

// For many rows: the tiled product of gemm_mfma.hip over an expert's run. A block of 8 waves works 128 rows of one run
// x 128 columns, a wave 32 x 64 as two tiles of the 32x32x16 instruction; K advances in steps of 64 through two buffers
// in shared memory (while a step's products run out of one, the next step's operands go from registers into the other
// and the step after that travels from memory to registers; one barrier a step; rows padded by 16 bytes against bank
// conflicts). A's rows are gathered through the run's pairs, and the results go to the pairs' own rows.
// Blocks with consecutive numbers go to different XCDs, each with a second-level cache of its own. An XCD takes one
// stretch of an order that walks panels of ET_PANEL row tiles column by column, so that the blocks it holds at a time
// form a rectangle and share their rows of A and of W (which are mostly one expert's); the stretches are cut from the
// tiles that exist, not from the most that could, so that all XCDs get as many.
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x16_t __attribute__((ext_vector_type(16)));
#define ET_BM 128
#define ET_BN 128
#define ET_BK 64
#define ET_LD (ET_BK + 8)
#define ET_PANEL 8
template <typename TO>
__global__ __launch_bounds__(512) void expert_gemm_tiled_kernel(const bf16_t* __restrict__ A, long lda, int a_div,
                                                                 const bf16_t* __restrict__ W, int N, int K,
                                                                 const int* __restrict__ offsets,
                                                                 const int* __restrict__ sorted, int E, int n_rows,
                                                                 TO* __restrict__ out, long ldo, int act, int gate_act, float limit,
                                                                   float shift, RowFactors rf) {
  constexpr int NT = 512, NA = ET_BM * 8 / NT, NWC = ET_BN * 8 / NT;
  __shared__ __attribute__((aligned(16))) bf16_t As[2][ET_BM][ET_LD];
  __shared__ __attribute__((aligned(16))) bf16_t Ws[2][ET_BN][ET_LD];
  __shared__ int rows[ET_BM];
  __shared__ float f_in[ET_BM], f_out[ET_BM];
  int n_tiles = 0;
  if (offsets)
    for (int i = 0; i < E; ++i) n_tiles += (offsets[i + 1] - offsets[i] + ET_BM - 1) / ET_BM;
  else
    n_tiles = (n_rows + ET_BM - 1) / ET_BM;
  const int col_tiles = (N + ET_BN - 1) / ET_BN, total = n_tiles * col_tiles;
  const int per_xcd = (total + 7) / 8, at = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per_xcd || at >= total) return;
  const int panel = at / (ET_PANEL * col_tiles), in_panel = at - panel * ET_PANEL * col_tiles;
  const int height = min(ET_PANEL, n_tiles - panel * ET_PANEL);
  int e, lo, hi;
  if (!expert_tile(offsets, E, n_rows, ET_BM, panel * ET_PANEL + in_panel % height, &e, &lo, &hi)) return;
  const int m = hi - lo < ET_BM ? hi - lo : ET_BM;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  if (tid < ET_BM) {
    const int row = tid < m ? (sorted ? sorted[lo + tid] : lo + tid) : -1;
    rows[tid] = row;
    factors_here(rf, row, &f_in[tid], &f_out[tid]);
  }
  __syncthreads();
  const int wm = wave / 2, wn = wave % 2;
  const int lr = lane & 31, lh = lane >> 5;
  const int n0 = in_panel / height * ET_BN;
  const bf16_t* We = W + (long)e * N * K;
  // every load is unconditional: rows beyond the run read the run's first row, columns beyond N the last one,
  // and their results are dropped
  long aoff[NA], woff[NWC];
  int arow_s[NA], wrow_s[NWC];
  const int scol = (tid & 7) * 8;
#pragma unroll
  for (int i = 0; i < NA; ++i) {
    arow_s[i] = (tid + NT * i) >> 3;
    const int src = rows[arow_s[i]] >= 0 ? rows[arow_s[i]] : rows[0];
    aoff[i] = (long)(src / a_div) * lda;
  }
#pragma unroll
  for (int i = 0; i < NWC; ++i) {
    wrow_s[i] = (tid + NT * i) >> 3;
    woff[i] = (long)min(n0 + wrow_s[i], N - 1) * K;
  }
  const bf16x8_t zero = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8_t ra[NA], rw[NWC];
  bool r_ok = false;
  auto fetch = [&](int k0) {
    const int kf = min(k0, K - 8);                     // the step after the last one reads the last again
    r_ok = k0 + scol < K;
    const int col = min(scol, K - 8 - kf);
#pragma unroll
    for (int i = 0; i < NA; ++i) ra[i] = *(const bf16x8_t*)(A + aoff[i] + kf + col);
#pragma unroll
    for (int i = 0; i < NWC; ++i) rw[i] = *(const bf16x8_t*)(We + woff[i] + kf + col);
  };
  auto store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NA; ++i) *(bf16x8_t*)&As[buf][arow_s[i]][scol] = r_ok ? ra[i] : zero;
#pragma unroll
    for (int i = 0; i < NWC; ++i) *(bf16x8_t*)&Ws[buf][wrow_s[i]][scol] = r_ok ? rw[i] : zero;
  };
  f32x16_t acc[2];
#pragma unroll
  for (int jn = 0; jn < 2; ++jn)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[jn][v] = 0.f;
  const int arow = wm * 32 + lr, wrow0 = wn * 64 + lr, wrow1 = wn * 64 + 32 + lr;
  fetch(0);
  store(0);
  fetch(ET_BK);
  __syncthreads();
  int buf = 0;
  for (int k0 = 0; k0 < K; k0 += ET_BK, buf ^= 1) {
#pragma unroll
    for (int kk = 0; kk < ET_BK / 16; ++kk) {
      const int kc = kk * 16 + lh * 8;
      const bf16x8_t b0 = *(const bf16x8_t*)&Ws[buf][wrow0][kc];
      const bf16x8_t b1 = *(const bf16x8_t*)&Ws[buf][wrow1][kc];
      const bf16x8_t a = *(const bf16x8_t*)&As[buf][arow][kc];
      acc[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b0, acc[0], 0, 0, 0);
      acc[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b1, acc[1], 0, 0, 0);
      if (kk == 0) {
        __builtin_amdgcn_sched_barrier(0);
        if (k0 + ET_BK < K) store(buf ^ 1);
        fetch(k0 + 2 * ET_BK);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
    __syncthreads();
  }
  // a lane holds C[row(v)][col]: row(v) = 8 * (v / 4) + 4 * (lane / 32) + v % 4 inside a 32 x 32 tile, col = lane % 32
#pragma unroll
  for (int v = 0; v < 16; ++v) {
    const int r = wm * 32 + (v >> 2) * 8 + lh * 4 + (v & 3), row = rows[r];
#pragma unroll
    for (int tn = 0; tn < 2; ++tn) {
      const int n = n0 + wn * 64 + tn * 32 + lr;
      expert_store<TO>(out, ldo, row, n, row >= 0 && n < N, acc[tn][v], act, gate_act, limit, shift, f_in[r], f_out[r]);
    }
  }
}

extern "C" int gl3_expert_gemm(const void* A, int a_dtype, long lda, int a_div, const void* W, int w_dtype, int E, int N, int K,
                               const int* offsets, const int* sorted, int n_rows, void* out, int out_dtype, long ldo, int act,
                               int use_mfma, int gate_act, float limit, float shift, const float* row_in, const float* row_out,
                               hipStream_t stream) {
  const RowFactors rf{row_in, row_out};
  if (n_rows == 0) return 0;
  GL3_REQUIRE(A && W && out && n_rows > 0 && E >= 1 && N > 0 && K > 0 && a_div >= 1 && lda >= K &&
                  ldo >= (gate_act >= 0 ? N / 2 : N),
              "gl3_expert_gemm: bad arguments");
  GL3_REQUIRE(gate_act < 0 || (GL3_ACT_KNOWN(gate_act) && N % 2 == 0),
              "gl3_expert_gemm: a gated expert has gate and up rows in turns (%d rows) and a known activation (%d)", N, gate_act);
  GL3_REQUIRE((offsets == nullptr) == (sorted == nullptr) && (offsets || E == 1),
              "gl3_expert_gemm: runs and their pairs come together; without them one expert takes every row");
  GL3_REQUIRE(act >= 0 && act <= 3, "gl3_expert_gemm: unknown activation %d", act);
  GL3_REQUIRE((N + 63) / 64 <= 65535, "gl3_expert_gemm: %d columns exceed the grid", N);
  const int e_eff = offsets ? E : 1;
  // (a product of a few columns, a router's: tiles of 128 columns would leave most of the chip idle; it takes the kernel
  // for few rows whatever its rows, in tiles of 16 of them)
  const bool narrow = !offsets && N <= 64;
  // many rows (an expert's run fills tiles of 128): the tiled kernel
  if (use_mfma && a_dtype == GL3_BF16 && w_dtype == GL3_BF16 && K % 8 == 0 && K >= 8 && lda % 8 == 0 &&
      (reinterpret_cast<uintptr_t>(A) % 16 == 0) && (reinterpret_cast<uintptr_t>(W) % 16 == 0) &&
      n_rows > 64 * e_eff && !narrow && (out_dtype == GL3_BF16 || out_dtype == GL3_F32)) {
    const long most = ((long)(n_rows + ET_BM - 1) / ET_BM + (offsets ? E : 0)) * ((N + ET_BN - 1) / ET_BN);
    GL3_REQUIRE(most < (1L << 30), "gl3_expert_gemm: %ld tiles exceed the grid", most);
    const dim3 grid((unsigned)((most + 7) / 8 * 8)), block(512);
    if (out_dtype == GL3_BF16)
      expert_gemm_tiled_kernel<bf16_t><<<grid, block, 0, stream>>>((const bf16_t*)A, lda, a_div, (const bf16_t*)W, N, K, offsets,
                                                                   sorted, E, n_rows, (bf16_t*)out, ldo, act, gate_act, limit, shift, rf);
    else
      expert_gemm_tiled_kernel<float><<<grid, block, 0, stream>>>((const bf16_t*)A, lda, a_div, (const bf16_t*)W, N, K, offsets,
                                                                  sorted, E, n_rows, (float*)out, ldo, act, gate_act, limit, shift, rf);
    GL3_LAUNCH_CHECK();
    return 0;
  }
  // few rows (an expert's run is a tile or two): the kernel that reads each weight row in long pieces, K in slices
  if (use_mfma && a_dtype == GL3_BF16 && w_dtype == GL3_BF16 && K % 8 == 0 && lda % 8 == 0 &&
      (reinterpret_cast<uintptr_t>(A) % 16 == 0) && (reinterpret_cast<uintptr_t>(W) % 16 == 0) &&
      (narrow || n_rows <= 64 * e_eff) && (N + EF_TN - 1) / EF_TN <= 65535 && (out_dtype == GL3_BF16 || out_dtype == GL3_F32)) {
    const int G = n_rows <= 16 * e_eff || narrow ? 1 : n_rows <= 32 * e_eff ? 2 : 4;      // by the runs' mean length
    const dim3 grid((n_rows + 16 * G - 1) / (16 * G) + (offsets ? E : 0), (N + EF_TN - 1) / EF_TN), block(EF_WAVES * 64);
#define EF_LAUNCH(TO, G)                                                                                                \
  expert_gemm_few_kernel<TO, G><<<grid, block, 0, stream>>>((const bf16_t*)A, lda, a_div, (const bf16_t*)W, N, K, offsets, \
                                                            sorted, E, n_rows, (TO*)out, ldo, act, gate_act, limit, shift, rf)
    if (out_dtype == GL3_BF16) {
      if (G == 1) EF_LAUNCH(bf16_t, 1); else if (G == 2) EF_LAUNCH(bf16_t, 2); else EF_LAUNCH(bf16_t, 4);
    } else {
      if (G == 1) EF_LAUNCH(float, 1); else if (G == 2) EF_LAUNCH(float, 2); else EF_LAUNCH(float, 4);
    }
#undef EF_LAUNCH
    GL3_LAUNCH_CHECK();
    return 0;
  }
  if (use_mfma && a_dtype == GL3_BF16 && w_dtype == GL3_BF16 && K % 16 == 0 && lda % 4 == 0 &&
      (reinterpret_cast<uintptr_t>(A) % 8 == 0) && (reinterpret_cast<uintptr_t>(W) % 8 == 0)) {
    const dim3 grid((n_rows + EM_TM - 1) / EM_TM + (offsets ? E : 0), (N + EM_TN - 1) / EM_TN), block(256);
    if (out_dtype == GL3_BF16)
      expert_gemm_mfma_kernel<bf16_t><<<grid, block, 0, stream>>>((const bf16_t*)A, lda, a_div, (const bf16_t*)W, N, K, offsets,
                                                                  sorted, E, n_rows, (bf16_t*)out, ldo, act, gate_act, limit, shift, rf);
    else if (out_dtype == GL3_F32)
      expert_gemm_mfma_kernel<float><<<grid, block, 0, stream>>>((const bf16_t*)A, lda, a_div, (const bf16_t*)W, N, K, offsets,
                                                                 sorted, E, n_rows, (float*)out, ldo, act, gate_act, limit, shift, rf);
    else GL3_REQUIRE(false, "gl3_expert_gemm: unknown output dtype %d", out_dtype);
    GL3_LAUNCH_CHECK();
    return 0;
  }
  const dim3 grid((n_rows + EG_TM - 1) / EG_TM + (offsets ? E : 0), (N + EG_TN - 1) / EG_TN), block(256);
#define EG_LAUNCH(TA, TW, TO)                                                                                          \
  expert_gemm_generic_kernel<TA, TW, TO><<<grid, block, 0, stream>>>((const TA*)A, lda, a_div, (const TW*)W, N, K, offsets, \
                                                                     sorted, E, n_rows, (TO*)out, ldo, act, gate_act, limit, shift, rf)
  if (a_dtype == GL3_F32 && w_dtype == GL3_F32 && out_dtype == GL3_F32) EG_LAUNCH(float, float, float);
  else if (a_dtype == GL3_BF16 && w_dtype == GL3_BF16 && out_dtype == GL3_BF16) EG_LAUNCH(bf16_t, bf16_t, bf16_t);
  else if (a_dtype == GL3_BF16 && w_dtype == GL3_BF16 && out_dtype == GL3_F32) EG_LAUNCH(bf16_t, bf16_t, float);
  else GL3_REQUIRE(false, "gl3_expert_gemm: dtypes %d x %d -> %d are not built", a_dtype, w_dtype, out_dtype);
#undef EG_LAUNCH
  GL3_LAUNCH_CHECK();
  return 0;
}

// ----------------------------------------------------------------- the weighted sum
// out[t] (+)= sum_j wts[t][j] * y[t * top + j], j in order. One thread an element. With idx [T][top] and n_real: a pair
// whose expert number is n_real or more is an identity expert, whose output is the token's input row h[t] itself (y
// holds nothing for it).
template <typename TH>
__global__ void route_combine_kernel(const float* __restrict__ y, const float* __restrict__ wts, int top, int d,
                                     float* __restrict__ out, int accumulate, long n, const int* __restrict__ idx,
                                     int n_real, const TH* __restrict__ h) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  const long t = i / d;
  const int c = i % d;
  float s = accumulate ? out[i] : 0.f;
  for (int j = 0; j < top; ++j) {
    const float v = (idx && idx[t * top + j] >= n_real) ? to_f32<TH>(h[t * d + c]) : y[(t * top + j) * d + c];
    s = fmaf(wts[t * top + j], v, s);
  }
  out[i] = s;
}

// The same, a block a row, for a step of few rows whose completed row a norm folded into the next product will read: also
// ssq[t] = the row's sum of squares and xg[t] = bfloat16(next_weight * row).
__global__ __launch_bounds__(1024) void route_combine_norm_kernel(const float* __restrict__ y, const float* __restrict__ wts,
                                                                   int top, int d, float* __restrict__ out,
                                                                   float* __restrict__ ssq,
                                                                   const float* __restrict__ next_weight,
                                                                   bf16_t* __restrict__ xg) {
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  float ss = 0.f;
  for (int c = threadIdx.x; c < d; c += blockDim.x) {
    float s = out[t * d + c];
    for (int j = 0; j < top; ++j) s = fmaf(wts[t * top + j], y[(t * top + j) * d + c], s);
    out[t * d + c] = s;
    xg[t * d + c] = static_cast<bf16_t>(next_weight[c] * s);
    ss += s * s;
  }
  ss = block_sum(ss, scratch);
  if (threadIdx.x == 0) ssq[t] = ss;
}

extern "C" int gl3_route_combine(const float* y, const float* wts, int n_tokens, int top, int d, float* out, int accumulate,
                                 const int* idx, int n_real, const void* h, int h_dtype, float* ssq,
                                 const float* next_weight, void* xg, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  GL3_REQUIRE(y && wts && out && n_tokens > 0 && top >= 1 && d > 0, "gl3_route_combine: bad arguments");
  GL3_REQUIRE((idx == nullptr) == (h == nullptr), "gl3_route_combine: identity experts need the choices and the input rows");
  const long n = (long)n_tokens * d;
  GL3_REQUIRE((n + 255) / 256 < (1L << 31), "gl3_route_combine: too many elements");
  GL3_REQUIRE((ssq == nullptr) == (next_weight == nullptr) && (ssq == nullptr) == (xg == nullptr) &&
                  (!ssq || (n_tokens <= 64 && accumulate && !idx)),
              "gl3_route_combine: what a folded norm reads comes together, for at most 64 rows that are added to");
  if (ssq) {
    const int threads = d >= 1024 ? 1024 : ((d + 63) / 64) * 64;
    route_combine_norm_kernel<<<dim3(n_tokens), dim3(threads), 0, stream>>>(y, wts, top, d, out, ssq, next_weight, (bf16_t*)xg);
    GL3_LAUNCH_CHECK();
    return 0;
  }
  if (h && h_dtype == GL3_BF16)
    route_combine_kernel<bf16_t><<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream>>>(y, wts, top, d, out, accumulate, n,
                                                                                            idx, n_real, (const bf16_t*)h);
  else
    route_combine_kernel<float><<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream>>>(y, wts, top, d, out, accumulate, n,
                                                                                           idx, n_real, (const float*)h);
  GL3_LAUNCH_CHECK();
  return 0;
}
