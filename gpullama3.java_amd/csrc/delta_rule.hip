// The gated delta rule: a mixer whose memory is one matrix per head instead of a cache of keys and values.
//
// Per value head h (reading key/query head h / (H / G)) and token, with S of size [D keys, Dv values] in 32-bit:
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// so the read-out sees the token's own write. q, k and v come out of a short causal convolution over time per
// channel (taps weights, the last one the current token's, zeros before a sequence's start) followed by silu; q and
// k are then scaled to unit length per head, x / sqrt(sum x^2 + unit_eps), and q by q_scale. The decay is
// g = exp(-exp(A_log[h]) softplus(a + dt_bias[h])), the write strength beta = sigmoid(b); a and b are two more
// columns per head of the same projection. Everything here is computed in 32-bit, with accurate exp and log.
//
// A sequence's state, one row of a [slots][state_stride] float array:
//   S in tiles of 16 value columns, [H][ceil(Dv / 16)][D][16] (a wave's share of S is consecutive memory),
//   then the convolution's last taps - 1 inputs of each of the C = 2 G D + H Dv channels, [C][taps - 1], oldest first.
// The tokens of a step are packed, sequence after sequence (cu_seqlens); each sequence is walked token by token from
// the state that earlier steps left, so a result does not depend on how the tokens were cut into steps.
//
// Two entry points: delta_prep (convolution, silu, unit length, decay and strength; then the convolution's new
// state) and delta_recurrence (the rule itself, then each head's read-out divided by its root mean square, times a
// weight shared by the heads, times silu or sigmoid of a gate).
//
// A decay per key channel instead of one per head: S <- diag(g) S, g of D numbers a head and token. delta_inner makes
// them, and the read-out's gate, from two-step projections: a of a key channel is its row of a second matrix times what a
// first one made of the input (a few numbers a token), and so is the gate.
#include "common.h"

__device__ __forceinline__ float dr_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float dr_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

struct DeltaShape {
  int H, G, D, Dv, taps;
  int ldp;            // floats a row of the projection
  int off_q, off_k, off_v, off_b, off_a;   // first column of each part in a row of the projection
  long state_stride;  // floats a slot
  long conv_off;      // where the convolution's inputs start in a slot's state
};

// grid (T, 2 G + H + 1): a q head, a k head, a v head, or the token's decays and strengths. One wave.
// one_each: every sequence of the step brings exactly one token (a decode step); the held inputs then move on here.
__global__ __launch_bounds__(64) void delta_prep_kernel(
    const float* __restrict__ proj, const float* __restrict__ conv_w, const float* __restrict__ A_log,
    const float* __restrict__ dt_bias, float* __restrict__ state, const int* __restrict__ cu_seqlens,
    const int* __restrict__ seq_of_token, const int* __restrict__ slot_ids, float* __restrict__ act,
    float* __restrict__ gates, DeltaShape s, float unit_eps, float q_scale, int one_each) {
  const int t = blockIdx.x, u = blockIdx.y, lane = threadIdx.x;
  const int C = 2 * s.G * s.D + s.H * s.Dv;
  const float* row = proj + (long)t * s.ldp;
  if (u == 2 * s.G + s.H) {
    for (int h = lane; h < s.H; h += 64) {
      if (A_log) {      // (null: the decays are per key channel and come from elsewhere)
        const float sp = dr_softplus(row[s.off_a + h] + dt_bias[h]);
        gates[(long)t * 2 * s.H + h] = expf(-expf(A_log[h]) * sp);
      }
      gates[(long)t * 2 * s.H + s.H + h] = dr_sigmoid(row[s.off_b + h]);
    }
    return;
  }
  const int b = seq_of_token[t];
  const int first = cu_seqlens[b], i = t - first;
  float* held = state + (long)slot_ids[b] * s.state_stride + s.conv_off;
  // the unit's channels: c0 .. c0 + n of the C convolved channels, which are columns col0 .. of the projection
  int c0, col0, n;
  if (u < s.G) { c0 = u * s.D; col0 = s.off_q + u * s.D; n = s.D; }
  else if (u < 2 * s.G) { c0 = s.G * s.D + (u - s.G) * s.D; col0 = s.off_k + (u - s.G) * s.D; n = s.D; }
  else { c0 = 2 * s.G * s.D + (u - 2 * s.G) * s.Dv; col0 = s.off_v + (u - 2 * s.G) * s.Dv; n = s.Dv; }
  const bool unit = u < 2 * s.G;
  float ss = 0.f;
  for (int e = lane; e < n; e += 64) {
    const int c = c0 + e;
    float y = 0.f;
    for (int r = 0; r < s.taps; ++r) {
      const int src = i - (s.taps - 1 - r);
      const float x = src >= 0 ? proj[(long)(first + src) * s.ldp + col0 + e] : held[(long)c * (s.taps - 1) + src + s.taps - 1];
      y = fmaf(conv_w[(long)c * s.taps + r], x, y);
    }
    y = y * dr_sigmoid(y);
    ss = fmaf(y, y, ss);
    act[(long)t * C + c] = y;
    if (one_each && s.taps > 1) {
      // every sequence brings one token: this lane is the only reader of the channel's held inputs, and moves them on
      float* hc = held + (long)c * (s.taps - 1);
      for (int jj = 0; jj + 2 < s.taps; ++jj) hc[jj] = hc[jj + 1];
      hc[s.taps - 2] = proj[(long)t * s.ldp + col0 + e];
    }
  }
  if (!unit) return;
  ss = wave_sum(ss);
  const float f = (u < s.G ? q_scale : 1.0f) / sqrtf(ss + unit_eps);
  for (int e = lane; e < n; e += 64) act[(long)t * C + c0 + e] *= f;   // (the lane's own stores of above)
}

// grid (B, ceil(C / 256)): a thread moves one channel's held inputs on by the sequence's new tokens, oldest first,
// so that no place is written before it has been read.
__global__ __launch_bounds__(256) void delta_conv_state_kernel(const float* __restrict__ proj, float* __restrict__ state,
                                                               const int* __restrict__ cu_seqlens,
                                                               const int* __restrict__ slot_ids, DeltaShape s) {
  const int b = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  const int GD = s.G * s.D, C = 2 * GD + s.H * s.Dv;
  if (c >= C) return;
  const int first = cu_seqlens[b], n = cu_seqlens[b + 1] - first;
  if (n <= 0) return;
  const int col = c < GD ? s.off_q + c : c < 2 * GD ? s.off_k + (c - GD) : s.off_v + (c - 2 * GD);
  float* held = state + (long)slot_ids[b] * s.state_stride + s.conv_off + (long)c * (s.taps - 1);
  for (int j = 0; j < s.taps - 1; ++j) {
    const int src = n - (s.taps - 1) + j;
    held[j] = src >= 0 ? proj[(long)(first + src) * s.ldp + col] : held[j + n];
  }
}

// The rule itself and the read-out's norm. grid (H, B, blocks a head: more than one where the launcher deals a prompt's head
// out), a wave owns 64 / RG value columns of head h's matrix, lane (r, c) of it the rows r, r + RG, ... of column c (RPL rows a
// lane), so a token costs a lane RPL multiply-adds for each of S^T k, the update and S^T q, and the sums over the lanes of
// a column are lane moves (no trip through shared memory). The tokens' operands (k, q, v, decays, strength) come in chunks
// of DR_CHUNK tokens through shared memory, the next chunk's loads on their way while the current chunk is worked on: what a
// token waits for is a wave's own instructions, not memory.
// Steps of few tokens: after the last token the block divides each of its tokens' read-outs (which it wrote to `o` itself) by
// their root mean square over the head and applies the weight and the gate: y = o / rms * w * silu(gate).
#define DR_CHUNK 16   // the most tokens a chunk; the launcher takes fewer where keys and values are long
#define DR_NLD 8       // loads a thread has on their way for the next chunk (with decays per channel DR_NLD_CH)
#define DR_NLD_CH 10

// Two sums at once over the RG lanes that share a column (lanes 64 / RG apart): both values travel together, p in the lower
// half of the wave and o in the upper, until both sums are in every lane. RG: the lanes a column's rows are dealt out to, 4, 8
// or 16 (16, 8 or 4 columns a wave; the state lies the same).
template <int RG>
__device__ __forceinline__ void dr_sum_pair(float& p, float& o) {
  auto a = __builtin_amdgcn_permlane32_swap(__float_as_uint(p), __float_as_uint(o), false, false);
  float x = __uint_as_float(a[0]) + __uint_as_float(a[1]);      // p over lanes l, l + 32; o the same in the upper half
  if (RG >= 8)    // lane l ^ 8 is 8 places round the row of 16
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));
  if (RG == 16)   // then lanes 8 apart hold the same: 4 places round the row are the other two
    x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x124, 0xf, 0xf, false));
  a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  a = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  p = __uint_as_float(a[0]);
  o = __uint_as_float(a[1]);
}

__device__ __forceinline__ float dr_gate(float z, int sigmoid) { return sigmoid ? dr_sigmoid(z) : z * dr_sigmoid(z); }

// CH: decay [T][H D] holds a factor per key channel, a third operand of D numbers beside k and q.
template <int RPL, typename TO, int MAXT, int RG, bool CH>
__global__ __launch_bounds__(MAXT) void delta_recurrence_kernel(
    const float* __restrict__ act, const float* __restrict__ gates, const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ cu_seqlens, const int* __restrict__ slot_ids, float* __restrict__ o,
    const float* __restrict__ proj, int ldp, int off_gate, const float* __restrict__ norm_w, TO* __restrict__ y,
    float eps, DeltaShape s, int chunk, int norm_here, int own_waves, int gate_sigmoid) {
  constexpr int NLD = CH ? DR_NLD_CH : DR_NLD;
  extern __shared__ __attribute__((aligned(16))) float dr_lds[];   // two buffers of chunk * per_token floats, and one token more
  typedef float f4 __attribute__((ext_vector_type(4)));
  const int h = blockIdx.x, b = blockIdx.y;
  constexpr int COLS = 64 / RG;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane / COLS, c = lane % COLS;
  const int D = s.D, H = s.H, Dv = s.Dv;
  // (a head's columns may be dealt out to several blocks, blockIdx.z: own_waves waves of columns each)
  const int j = ((int)blockIdx.z * own_waves + wave) * COLS + c;
  const bool valid = wave < own_waves && j < Dv;
  const int C = 2 * s.G * D + H * Dv;
  const int kvh = h / (H / s.G);
  const int first = cu_seqlens[b], last = cu_seqlens[b + 1];
  if (last <= first) return;
  const int CT = (Dv + 15) / 16;
  const bool owner = wave < own_waves && j < CT * 16;     // (a block may have more waves than columns to own: they only help to load)
  // the lane's column in the state's tiles of 16 columns: row i of it at [16 i]
  float* tile = state + (long)slot_ids[b] * s.state_stride + ((long)(h * CT + (owner ? j / 16 : 0)) * D) * 16 + (j & 15);
  float S[RPL];
#pragma unroll
  for (int ii = 0; ii < RPL; ++ii) {
    const int i = r + RG * ii;
    S[ii] = (owner && i < D) ? tile[(long)i * 16] : 0.f;
  }
  // A token's operands in a chunk's buffer: q | k (| decays) | v [Dv] | decay, strength, where q and k lie as the lanes read
  // them: row r + RG ii at [r][ii], RPL places a lane (rows beyond D stay zero), so a lane's share is 16-byte reads.
  constexpr int NV = CH ? 3 : 2;                                // vectors over the key channels
  const int per_src = NV * D + Dv + (CH ? 1 : 2);               // what a token brings
  constexpr int VEC = RG * RPL;                                 // places of q, and of k
  const int per_token = NV * VEC + ((Dv + 2 + 3) & ~3);         // what it takes in the buffer
  const int n_src = chunk * per_src;
  const long q_at = (long)kvh * D, k_at = (long)s.G * D + (long)kvh * D, v_at = 2L * s.G * D + (long)h * Dv;
  const int threads = blockDim.x;
  for (int e = tid; e < (2 * chunk + 1) * per_token; e += threads) dr_lds[e] = 0.f;      // (one token more: see the reads ahead)
  __syncthreads();
  // This thread's places: place n of a chunk is operand e = tid + n threads of the chunk's per_src a token. Where it comes
  // from in the first chunk, how far that moves on from chunk to chunk, and where it goes are worked out once.
  float held[NLD] = {};
  const float* from[NLD];
  int step[NLD], to[NLD];
#pragma unroll
  for (int n = 0; n < NLD; ++n) {
    const int e = tid + n * threads;
    const int tt = e / per_src, f = e - tt * per_src;
    const long t = first + tt;
    int at;
    if (f < NV * D) {
      const int which = CH && f >= 2 * D ? 2 : f >= D, i = f - which * D;
      at = which * VEC + (i % RG) * RPL + i / RG;
      from[n] = which == 2 ? decay + t * H * D + (long)h * D + i : act + t * C + (which ? k_at : q_at) + i;
      step[n] = (which == 2 ? H * D : C) * chunk;
    } else {
      at = NV * VEC + (f - NV * D);
      const bool value = f < NV * D + Dv;
      from[n] = value ? act + t * C + v_at + (f - NV * D) : gates + t * 2 * H + (long)(CH ? 1 : f - 2 * D - Dv) * H + h;
      step[n] = (value ? C : 2 * H) * chunk;
    }
    to[n] = tt * per_token + at;
  }
  auto ask = [&](int t0) {      // (called for one chunk after the other)
    const int here = min(n_src, (last - t0) * per_src);
#pragma unroll
    for (int n = 0; n < NLD; ++n) {
      if (tid + n * threads < here) held[n] = *from[n];
      from[n] += step[n];
    }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int n = 0; n < NLD; ++n)
      if (tid + n * threads < n_src) dr_lds[buf * chunk * per_token + to[n]] = held[n];
  };
  ask(first);
  put(0);
  __syncthreads();
  // A token's read-out is made in the pass of the token after it, with the matrix as it stands then: its sum over the rows
  // and the next token's S^T k are one reduction. So a pass takes k, decay, v and strength of its own token and q of the one
  // before (zeros for the first: the buffers were cleared), and stores the read-out of the one before.
  struct Operands { float k[RPL], q[RPL], gs[CH ? RPL : 1], v, beta; };
  const int lane_at = r * RPL, v_place = NV * VEC + (valid ? j : 0);
  auto fetch = [&](Operands& x, int at, int q_from) {      // (places of the token's operands, and of the token's before it)
    const float *op = dr_lds + at, *oq = dr_lds + q_from + lane_at;
#pragma unroll
    for (int ii = 0; ii < RPL; ii += 4) {
      const f4 q4 = *(const f4*)(oq + ii), k4 = *(const f4*)(op + lane_at + VEC + ii);
#pragma unroll
      for (int e = 0; e < 4; ++e) { x.q[ii + e] = q4[e]; x.k[ii + e] = k4[e]; }
      if constexpr (CH) {
        const f4 g4 = *(const f4*)(op + lane_at + 2 * VEC + ii);
#pragma unroll
        for (int e = 0; e < 4; ++e) x.gs[ii + e] = g4[e];
      }
    }
    if constexpr (!CH) x.gs[0] = op[NV * VEC + Dv];
    x.beta = op[NV * VEC + Dv + (CH ? 0 : 1)];
    x.v = op[v_place];
  };
  float* read_out = o + (long)first * H * Dv + (long)h * Dv + j;
  int advance = 0;                       // (the first pass has no read-out to store: its zero lands where the second's goes)
  const bool whole = __all(valid);
  auto store = [&](float v) {            // (all lanes of a column hold the same number)
    if (whole) *read_out = v;
    else if (valid) *read_out = v;
    read_out += advance;
    advance = H * Dv;
  };
  auto work = [&](const Operands& x) {
    float p2[2] = {0.f, 0.f}, o2[2] = {0.f, 0.f};
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii) {
      o2[ii & 1] = fmaf(S[ii], x.q[ii], o2[ii & 1]);
      S[ii] *= x.gs[CH ? ii : 0];
      p2[ii & 1] = fmaf(S[ii], x.k[ii], p2[ii & 1]);
    }
    float part = p2[0] + p2[1], read = o2[0] + o2[1];
    dr_sum_pair<RG>(part, read);
    const float uu = valid ? x.beta * (x.v - part) : 0.f;
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii) S[ii] = fmaf(x.k[ii], uu, S[ii]);
    store(read);
  };
  int buf = 0, q_last = (2 * chunk - 1) * per_token;
  for (int t0 = first; t0 < last; t0 += chunk) {
    const bool more = t0 + chunk < last;
    if (more) ask(t0 + chunk);
    const int n_here = min(chunk, last - t0);
    int at = buf * chunk * per_token;
    Operands xa;
    fetch(xa, at, q_last);
    if constexpr (RPL <= (CH ? 16 : 24) && MAXT <= 512) {
      // (two tokens' operands in registers in turn: the next token's reads from shared memory are on their way while the
      // current token's chain of multiply-adds runs; the read behind a chunk's last token is of no use and does no harm)
      Operands xb;
      int tt = 0;
      for (; tt + 2 <= n_here; tt += 2) {
        fetch(xb, at + per_token, at);
        work(xa);
        fetch(xa, at + 2 * per_token, at + per_token);
        work(xb);
        at += 2 * per_token;
      }
      if (tt < n_here) {
        work(xa);
        at += per_token;
      }
    } else {                              // (long keys, or a block of sixteen waves: two tokens' operands beside the matrix do not fit the registers)
      for (int tt = 0; tt < n_here; ++tt) {
        if (tt > 0) fetch(xa, at, at - per_token);
        work(xa);
        at += per_token;
      }
    }
    q_last = at - per_token;              // (the next chunk is put beside this one, not over it)
    if (more) put(buf ^ 1);
    __syncthreads();
    buf ^= 1;
  }
  {                                       // the last token's read-out
    float read = 0.f, none = 0.f;
#pragma unroll
    for (int ii = 0; ii < RPL; ++ii) read = fmaf(S[ii], dr_lds[q_last + lane_at + ii], read);
    dr_sum_pair<RG>(none, read);
    store(read);
  }
#pragma unroll
  for (int ii = 0; ii < RPL; ++ii) {
    const int i = r + RG * ii;
    if (owner && i < D) tile[(long)i * 16] = S[ii];
  }
  // (steps of many tokens a sequence: a launch of its own, with a wave to every token and head, normalises them)
  if (!norm_here) return;
  // the read-outs of this head are all this block's own stores: made visible to its other waves, then normalised
  __threadfence_block();
  __syncthreads();
  const int n_waves = threads >> 6;
  for (int t = first + wave; t < last; t += n_waves) {
    const float* orow = o + ((long)t * H + h) * Dv;
    const float* grow = proj + (long)t * ldp + off_gate + (long)h * Dv;
    float ss = 0.f;
    for (int e = lane; e < Dv; e += 64) {
      const float x = orow[e];
      ss = fmaf(x, x, ss);
    }
    ss = wave_sum(ss);
    const float f = 1.0f / sqrtf(ss / (float)Dv + eps);
    TO* dst = y + ((long)t * H + h) * Dv;
    for (int e = lane; e < Dv; e += 64) {
      const float z = grow[e];
      dst[e] = from_f32<TO>(orow[e] * f * norm_w[e] * dr_gate(z, gate_sigmoid));
    }
  }
}

// The same for a step in which every sequence brings ONE token: the time is the matrices' way from memory and back. A block
// a (head, sequence), a wave a tile of 16 columns; lane (r, c) holds 4 consecutive columns 4 c of the rows r, r + 16, ... (16
// bytes each, a wave 1 KB of consecutive memory), and reads its rows' operands straight from memory. At the end the block
// norms the head's read-outs, which stay in shared memory. IT: 16ths of the rows, rounded up.
template <int IT, typename TO, bool CH>
__global__ __launch_bounds__(1024) void delta_one_token_kernel(
    const float* __restrict__ act, const float* __restrict__ gates, const float* __restrict__ decay, float* __restrict__ state,
    const int* __restrict__ slot_ids, const float* __restrict__ proj, int ldp, int off_gate, const float* __restrict__ norm_w,
    TO* __restrict__ y, float eps, DeltaShape s, int gate_sigmoid) {
  typedef float f4 __attribute__((ext_vector_type(4)));
  __shared__ float read[256];
  __shared__ float scratch[16];
  const int h = blockIdx.x, t = blockIdx.y, tile = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane >> 2, c = (lane & 3) * 4;
  const int D = s.D, H = s.H, Dv = s.Dv, C = 2 * s.G * D + H * Dv, CT = (Dv + 15) / 16;
  float* mat = state + (long)slot_ids[t] * s.state_stride + ((long)(h * CT + tile) * D) * 16 + c;
  const float* row = act + (long)t * C;
  const float* qp = row + (long)(h / (H / s.G)) * D;
  const float* kp = qp + (long)s.G * D;
  f4 S[IT];
  float k[IT], q[IT], g[CH ? IT : 1];
#pragma unroll
  for (int n = 0; n < IT; ++n) {
    const int i = r + 16 * n;
    const bool ok = i < D;
    S[n] = ok ? *(const f4*)(mat + (long)i * 16) : f4{0.f, 0.f, 0.f, 0.f};
    k[n] = ok ? kp[i] : 0.f;
    q[n] = ok ? qp[i] : 0.f;
    if (CH) g[n] = ok ? decay[(long)t * H * D + (long)h * D + i] : 0.f;
  }
  if (!CH) g[0] = gates[(long)t * 2 * H + h];
  const float beta = gates[(long)t * 2 * H + H + h];
  float v[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = tile * 16 + c + e < Dv ? row[2L * s.G * D + (long)h * Dv + tile * 16 + c + e] : 0.f;
  auto over_rows = [](f4 p) {            // the sum over the 16 lanes that hold the same columns
#pragma unroll
    for (int o = 4; o < 64; o <<= 1)
#pragma unroll
      for (int e = 0; e < 4; ++e) p[e] += __shfl_xor(p[e], o, 64);
    return p;
  };
  f4 p = {0.f, 0.f, 0.f, 0.f}, out = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int n = 0; n < IT; ++n) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      S[n][e] *= g[CH ? n : 0];
      p[e] = fmaf(S[n][e], k[n], p[e]);
    }
  }
  p = over_rows(p);
  float u[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) u[e] = beta * (v[e] - p[e]);
#pragma unroll
  for (int n = 0; n < IT; ++n) {
    const int i = r + 16 * n;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      S[n][e] = fmaf(k[n], u[e], S[n][e]);
      out[e] = fmaf(S[n][e], q[n], out[e]);
    }
    if (i < D) *(f4*)(mat + (long)i * 16) = S[n];
  }
  out = over_rows(out);
  if (r == 0) {
#pragma unroll
    for (int e = 0; e < 4; ++e) read[tile * 16 + c + e] = out[e];
  }
  __syncthreads();
  const int j = threadIdx.x;
  const float o = j < Dv ? read[j] : 0.f;
  const float f = 1.0f / sqrtf(block_sum(o * o, scratch) / (float)Dv + eps);
  if (j < Dv) {
    const float z = proj[(long)t * ldp + off_gate + (long)h * Dv + j];
    y[((long)t * H + h) * Dv + j] = from_f32<TO>(o * f * norm_w[j] * dr_gate(z, gate_sigmoid));
  }
}

// grid (T, H), one wave: y[t, h, :] = o / sqrt(mean(o^2) + eps) * w * silu(gate[t, h, :]) (or sigmoid of it)
template <typename TO>
__global__ __launch_bounds__(64) void delta_gated_norm_kernel(const float* __restrict__ o, const float* __restrict__ proj,
                                                              int ldp, int off_gate, const float* __restrict__ w,
                                                              TO* __restrict__ y, int H, int Dv, float eps,
                                                              int gate_sigmoid) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const float* orow = o + ((long)t * H + h) * Dv;
  const float* grow = proj + (long)t * ldp + off_gate + (long)h * Dv;
  float ss = 0.f;
  for (int e = lane; e < Dv; e += 64) ss = fmaf(orow[e], orow[e], ss);
  ss = wave_sum(ss);
  const float f = 1.0f / sqrtf(ss / (float)Dv + eps);
  TO* dst = y + ((long)t * H + h) * Dv;
  for (int e = lane; e < Dv; e += 64) {
    const float z = grow[e];
    dst[e] = from_f32<TO>(orow[e] * f * w[e] * dr_gate(z, gate_sigmoid));
  }
}

static int delta_shape(DeltaShape& s, int H, int G, int D, int Dv, int taps, int ldp, int off_q, int off_k, int off_v,
                       int off_b, int off_a, long state_stride) {
  GL3_REQUIRE(H > 0 && G > 0 && H % G == 0 && D > 0 && D <= 256 && Dv > 0 && taps >= 1 && taps <= 64,
              "delta rule: %d heads over %d key heads of %d, values of %d, %d taps", H, G, D, Dv, taps);
  const long CT = (Dv + 15) / 16, C = 2L * G * D + (long)H * Dv;
  s = DeltaShape{H, G, D, Dv, taps, ldp, off_q, off_k, off_v, off_b, off_a, state_stride, (long)H * CT * D * 16};
  GL3_REQUIRE(state_stride >= s.conv_off + C * (taps - 1), "delta rule: a slot's state of %ld floats is too small",
              state_stride);
  const int ends[5] = {off_q + G * D, off_k + G * D, off_v + H * Dv, off_b + H, off_a + H};
  for (int i = 0; i < 5; ++i) GL3_REQUIRE(ends[i] <= ldp, "delta rule: the projection's rows of %d are too short", ldp);
  GL3_REQUIRE(off_q >= 0 && off_k >= 0 && off_v >= 0 && off_b >= 0 && off_a >= 0, "delta rule: a negative column");
  return 0;
}

extern "C" long gl3_delta_state_floats(int H, int G, int D, int Dv, int taps) {
  return (long)H * ((Dv + 15) / 16) * D * 16 + (2L * G * D + (long)H * Dv) * (taps - 1);
}

// proj [T][ldp] float: the projection of the step's tokens. conv_w [C][taps], A_log [H], dt_bias [H] float.
// state [slots][state_stride] float. act [T][C] and gates [T][2 H] float are written; then the held inputs move on
// (one_each: the caller vouches that every sequence brings exactly one token, and they move on in the same launch).
// A_log and dt_bias null: no decays per head (gates then holds the strengths in its second half only).
extern "C" int gl3_delta_prep(const float* proj, const float* conv_w, const float* A_log, const float* dt_bias,
                              float* state, const int* cu_seqlens, const int* seq_of_token, const int* slot_ids,
                              float* act, float* gates, int T, int B, int H, int G, int D, int Dv, int taps, int ldp,
                              int off_q, int off_k, int off_v, int off_b, int off_a, long state_stride, float unit_eps,
                              float q_scale, int one_each, hipStream_t stream) {
  if (T == 0 || B == 0) return 0;
  GL3_REQUIRE(proj && conv_w && (A_log == nullptr) == (dt_bias == nullptr) && state && cu_seqlens && seq_of_token && slot_ids && act && gates &&
                  T > 0 && B > 0, "gl3_delta_prep: bad arguments");
  DeltaShape s;
  if (delta_shape(s, H, G, D, Dv, taps, ldp, off_q, off_k, off_v, off_b, off_a, state_stride)) return -1;
  GL3_REQUIRE(2 * G + H + 1 <= 65535 && B <= 65535, "gl3_delta_prep: too many heads or sequences for the grid");
  delta_prep_kernel<<<dim3(T, 2 * G + H + 1), dim3(64), 0, stream>>>(proj, conv_w, A_log, dt_bias, state, cu_seqlens,
                                                                     seq_of_token, slot_ids, act, gates, s, unit_eps, q_scale, one_each);
  GL3_LAUNCH_CHECK();
  GL3_REQUIRE(!one_each || T == B, "gl3_delta_prep: %d tokens of %d sequences are not one each", T, B);
  if (taps > 1 && !one_each) {
    const int C = 2 * G * D + H * Dv;
    delta_conv_state_kernel<<<dim3(B, (C + 255) / 256), dim3(256), 0, stream>>>(proj, state, cu_seqlens, slot_ids, s);
    GL3_LAUNCH_CHECK();
  }
  return 0;
}

// act [T][C], gates [T][2 H] as gl3_delta_prep left them. o [T][H Dv] float receives the raw read-outs (scratch);
// y [T][H Dv] (float or bfloat16) the read-outs divided by their root mean square over each head, times norm_w [Dv]
// (float), times silu of the gate (gate_sigmoid: sigmoid), whose H Dv columns start at off_gate of proj [T][ldp] (float).
// decay [T][H D] (may be null): a factor per key channel, in place of the heads' decays in gates. one_each: every sequence
// brings exactly one token (o is then left alone where the slots' states lie at multiples of 16 bytes).
extern "C" int gl3_delta_recurrence(const float* act, const float* gates, const float* decay, float* state, const int* cu_seqlens,
                                    const int* slot_ids, float* o, const float* proj, int ldp, int off_gate,
                                    const float* norm_w, void* y, int y_dtype, float eps, int T, int B, int H, int G, int D,
                                    int Dv, int taps, long state_stride, int gate_sigmoid, int one_each, hipStream_t stream) {
  if (B == 0 || T == 0) return 0;
  GL3_REQUIRE(act && gates && state && cu_seqlens && slot_ids && o && proj && norm_w && y && B > 0,
              "gl3_delta_recurrence: bad arguments");
  DeltaShape s;
  if (delta_shape(s, H, G, D, Dv, taps, 1 << 30, 0, 0, 0, 0, 0, state_stride)) return -1;
  GL3_REQUIRE(H <= 65535 && B <= 65535, "gl3_delta_recurrence: too many heads or sequences for the grid");
  GL3_REQUIRE(Dv <= 256, "gl3_delta_recurrence: values of %d elements: a block holds up to 256 columns", Dv);
  GL3_REQUIRE(off_gate >= 0 && off_gate + H * Dv <= ldp, "gl3_delta_recurrence: the gate's columns %d .. of rows of %d", off_gate, ldp);
  GL3_REQUIRE(y_dtype == GL3_F32 || y_dtype == GL3_BF16, "gl3_delta_recurrence: unknown dtype %d", y_dtype);
  GL3_REQUIRE(!one_each || T == B, "gl3_delta_recurrence: %d tokens of %d sequences are not one each", T, B);
  if (one_each && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0) {
    const dim3 grid1(H, B), block1((Dv + 15) / 16 * 64);
#define ONE3(IT, TO, CH)                                                                                                    \
  delta_one_token_kernel<IT, TO, CH><<<grid1, block1, 0, stream>>>(act, gates, decay, state, slot_ids, proj, ldp, off_gate, \
                                                                   norm_w, (TO*)y, eps, s, gate_sigmoid)
#define ONE2(IT, TO)                     \
  do {                                   \
    if (decay) ONE3(IT, TO, true);       \
    else ONE3(IT, TO, false);            \
  } while (0)
#define ONE(IT)                                  \
  do {                                           \
    if (y_dtype == GL3_F32) ONE2(IT, float);     \
    else ONE2(IT, bf16_t);                       \
  } while (0)
    if (D <= 32) ONE(2);
    else if (D <= 64) ONE(4);
    else if (D <= 128) ONE(8);
    else ONE(16);
#undef ONE
#undef ONE2
#undef ONE3
    GL3_LAUNCH_CHECK();
    return 0;
  }
  // as many waves as the columns need, and as the loads of a chunk of operands need (DR_NLD a thread)
  // the read-outs' norm: by the block that made them where a sequence brings few tokens (a decode step), else by a
  // launch of its own with a wave to every token and head (a block's few waves would walk a prompt's tokens one by one)
  const int norm_here = T <= 4 * B;
  // A prompt's chain of tokens is bound by a wave's instructions per token: the fewer rows a lane, the fewer of them (one
  // prompt of 2,048 tokens, 32 heads of 64 and decays per channel: 4 lanes a column 690 us, 8 lanes 500, 16 lanes 400), in blocks
  // of at most eight waves, a head's columns dealt out to several blocks (grid z) if need be. Where sequences enough run
  // side by side to fill the chip, 8 lanes: their total of instructions is less (eight sequences of 512 tokens: 176 against 200).
  // Steps of few tokens a sequence: 4 lanes, a block a head, which norms the head's read-outs itself.
  auto blocks_a_head = [&](int lanes) { return ((long)Dv * lanes + 64 * 8 - 1) / (64 * 8); };
  const int rg = norm_here || D < 32 ? 4 : D >= 48 && (long)H * B * blocks_a_head(16) <= 256 ? 16 : 8;
  const int cols = 64 / rg;
  const int all_col_waves = (Dv + cols - 1) / cols;
  const int want = norm_here ? 1 : (int)blocks_a_head(rg);
  const int col_waves = (all_col_waves + want - 1) / want;
  const int split = (all_col_waves + col_waves - 1) / col_waves;
  // (fewer tokens a chunk where that keeps the block at the waves its columns need, or at four)
  const int nv = decay ? 3 : 2, nld = decay ? DR_NLD_CH : DR_NLD, per_src = nv * D + Dv + (decay ? 1 : 2);
  int chunk = DR_CHUNK, waves = col_waves;
  const int rows = (D + rg - 1) / rg;
  const int rpl = rows <= 4 ? 4 : rows <= 8 ? 8 : rows <= 16 ? 16 : rows <= 24 ? 24 : rows <= 32 ? 32 : rows <= 48 ? 48 : 64;
  const size_t lds_token = (size_t)(nv * rg * rpl + ((Dv + 2 + 3) & ~3)) * sizeof(float);
  for (;; chunk /= 2) {
    waves = col_waves;
    while (waves * 64 * nld < chunk * per_src) ++waves;
    if ((waves <= (col_waves > 4 ? col_waves : 4) && (2 * chunk + 1) * lds_token <= 64 * 1024) || chunk == 1) break;
  }
  GL3_REQUIRE(waves <= 16, "gl3_delta_recurrence: keys of %d with values of %d need more than a block's threads", D, Dv);
  dim3 grid(H, B, split), block(waves * 64);
  const size_t lds = (2 * chunk + 1) * lds_token;
  GL3_REQUIRE(lds <= 64 * 1024, "gl3_delta_recurrence: a chunk's operands of %zu bytes exceed shared memory", lds);
#define GO5(R, TO, MAXT, RGV, CH)                                                                                          \
  delta_recurrence_kernel<R, TO, MAXT, RGV, CH><<<grid, block, lds, stream>>>(                                             \
      act, gates, decay, state, cu_seqlens, slot_ids, o, proj, ldp, off_gate, norm_w, (TO*)y, eps, s, chunk, norm_here,    \
      col_waves, gate_sigmoid)
#define GO4(R, TO, MAXT, RGV)                                                  \
  do {                                                                         \
    if (decay) GO5(R, TO, MAXT, RGV, true);                                    \
    else GO5(R, TO, MAXT, RGV, false);                                         \
  } while (0)
#define GO3(R, TO, MAXT)                                                       \
  do {                                                                         \
    if constexpr (R <= 16) {                                                   \
      if (rg == 16) { GO4(R, TO, MAXT, 16); break; }                           \
    }                                                                          \
    if constexpr (R <= 32) {                                                   \
      if (rg == 8) { GO4(R, TO, MAXT, 8); break; }                             \
    }                                                                          \
    GO4(R, TO, MAXT, 4);                                                       \
  } while (0)
#define GO2(R, TO)                                                             \
  do {                                                                         \
    if (waves <= 4) GO3(R, TO, 256);                                           \
    else if (waves <= 8) GO3(R, TO, 512);                                      \
    else GO3(R, TO, 1024);                                                     \
  } while (0)
#define GO(R)                                                                  \
  do {                                                                         \
    if (y_dtype == GL3_F32) GO2(R, float);                                     \
    else GO2(R, bf16_t);                                                       \
  } while (0)
  switch (rpl) {
    case 4: GO(4); break;
    case 8: GO(8); break;
    case 16: GO(16); break;
    case 24: GO(24); break;
    case 32: GO(32); break;
    case 48: GO(48); break;
    default: GO(64); break;
  }
#undef GO
#undef GO2
#undef GO3
#undef GO4
#undef GO5
  GL3_LAUNCH_CHECK();
  if (!norm_here) {
    GL3_REQUIRE(T <= 2147483647 / 64, "gl3_delta_recurrence: %d tokens exceed the grid", T);
    if (y_dtype == GL3_F32)
      delta_gated_norm_kernel<float><<<dim3(T, H), dim3(64), 0, stream>>>(o, proj, ldp, off_gate, norm_w, (float*)y, H, Dv, eps,
                                                                                 gate_sigmoid);
    else
      delta_gated_norm_kernel<bf16_t><<<dim3(T, H), dim3(64), 0, stream>>>(o, proj, ldp, off_gate, norm_w, (bf16_t*)y, H, Dv, eps,
                                                                                  gate_sigmoid);
  }
  GL3_LAUNCH_CHECK();
  return 0;
}

// ----------------------------------------------------------------- decays per key channel and the gate, two-step projections
// proj [T][ldp] float: the first steps' sums, ra columns from col_a (decays) and rg from col_g (gate). w2 [Na + Ng][Rp]: the
// second steps' rows, the decays' first (padded with zero rows to Na, a multiple of 64), then the gate's (padded to Ng, a
// multiple of 64), zeros behind each row's ra or rg numbers up to Rp, a multiple of 32.
//   decay [T][HD] = exp(-exp(A_log[n / D]) softplus(sum + dt_bias[n])),  gate [T][HV] = sum
// A block takes 64 columns of w2 for 16 MT tokens; the first steps' sums are rounded to the weights' type, as any
// product's input is.
struct DeltaInner {
  int ldp, col_a, ra, col_g, rg, Rp, Na, HD, HV, D, T;
};
// What a lane knows of its column n of w2; `store` takes the column's sum for token t. FAST: the hardware's exponential
// and logarithm (an error of some 1e-7 of numbers around one: 32-bit rounding of the decay itself).
struct InnerColumn {
  float rate, bias;
  float* out;
  long ld;
  bool is_decay, exists;
  __device__ __forceinline__ InnerColumn(int n, const DeltaInner& s, const float* A_log, const float* dt_bias, float* decay,
                                         float* gate) {
    is_decay = n < s.Na;
    exists = is_decay ? n < s.HD : n - s.Na < s.HV;
    ld = is_decay ? s.HD : s.HV;
    out = is_decay ? decay + n : gate + (n - s.Na);
    rate = is_decay && exists ? -expf(A_log[n / s.D]) : 0.f;
    bias = is_decay && exists ? dt_bias[n] : 0.f;
  }
  template <bool FAST>
  __device__ __forceinline__ void store(float v, int t, int T) const {
    if (!exists || t >= T) return;
    if (is_decay) {
      v += bias;
      if (FAST) {
        const float sp = v > 20.f ? v : 0.6931471805599453f * __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(1.4426950408889634f * v));
        v = __builtin_amdgcn_exp2f(1.4426950408889634f * rate * sp);
      } else {
        v = expf(rate * dr_softplus(v));
      }
    }
    out[(long)t * ld] = v;
  }
};

typedef __bf16 di_bf16x8 __attribute__((ext_vector_type(8)));
typedef float di_f32x4 __attribute__((ext_vector_type(4)));
template <int MT>
__global__ __launch_bounds__(256) void delta_inner_mfma_kernel(const float* __restrict__ proj, const bf16_t* __restrict__ w2,
                                                               const float* __restrict__ A_log, const float* __restrict__ dt_bias,
                                                               float* __restrict__ decay, float* __restrict__ gate, DeltaInner s) {
  extern __shared__ __attribute__((aligned(16))) char di_smem[];
  bf16_t* As = reinterpret_cast<bf16_t*>(di_smem);            // [16 MT][Rp + 8]
  const int lda = s.Rp + 8;
  const int n0 = blockIdx.x * 64, t0 = blockIdx.y * 16 * MT;
  const int col = n0 < s.Na ? s.col_a : s.col_g, r = n0 < s.Na ? s.ra : s.rg;
  for (int row = threadIdx.x >> 5; row < 16 * MT; row += 8)
    for (int k = threadIdx.x & 31; k < s.Rp; k += 32)
      As[row * lda + k] = static_cast<bf16_t>(k < r && t0 + row < s.T ? proj[(long)(t0 + row) * s.ldp + col + k] : 0.f);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, li = lane & 15, lq = lane >> 4;
  const int n = n0 + wave * 16 + li;
  const bf16_t* wp = w2 + (long)n * s.Rp + 8 * lq;
  const InnerColumn mine(n, s, A_log, dt_bias, decay, gate);
  di_f32x4 acc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) acc[m] = di_f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  for (int k = 0; k < s.Rp; k += 32) {
    const di_bf16x8 b = *reinterpret_cast<const di_bf16x8*>(wp + k);
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const di_bf16x8 a = *reinterpret_cast<const di_bf16x8*>(As + (16 * m + li) * lda + k + 8 * lq);
      acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[m], 0, 0, 0);
    }
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int i = 0; i < 4; ++i) mine.store<true>(acc[m][i], t0 + 16 * m + 4 * lq + i, s.T);
}

__global__ __launch_bounds__(256) void delta_inner_f32_kernel(const float* __restrict__ proj, const float* __restrict__ w2,
                                                              const float* __restrict__ A_log, const float* __restrict__ dt_bias,
                                                              float* __restrict__ decay, float* __restrict__ gate, DeltaInner s) {
  const int n = blockIdx.x * 64 + (threadIdx.x & 63), t = blockIdx.y * 4 + (threadIdx.x >> 6);
  if (t >= s.T) return;
  const int col = n < s.Na ? s.col_a : s.col_g, r = n < s.Na ? s.ra : s.rg;
  const float* a = proj + (long)t * s.ldp + col;
  const float* w = w2 + (long)n * s.Rp;
  float v = 0.f;
  for (int k = 0; k < r; ++k) v = fmaf(a[k], w[k], v);
  InnerColumn(n, s, A_log, dt_bias, decay, gate).store<false>(v, t, s.T);
}

extern "C" int gl3_delta_inner(const float* proj, int ldp, int col_a, int ra, int col_g, int rg, const void* w2, int w_dtype,
                               int Rp, int Na, int Ng, const float* A_log, const float* dt_bias, float* decay, float* gate,
                               int T, int H, int D, int Dv, hipStream_t stream) {
  if (T == 0) return 0;
  GL3_REQUIRE(proj && w2 && A_log && dt_bias && decay && gate && T > 0 && H > 0 && D > 0 && Dv > 0, "gl3_delta_inner: bad arguments");
  GL3_REQUIRE(ra > 0 && rg > 0 && Rp % 32 == 0 && ra <= Rp && rg <= Rp && Rp <= 1024, "gl3_delta_inner: inner sizes %d and %d in rows of %d",
              ra, rg, Rp);
  GL3_REQUIRE(col_a >= 0 && col_g >= 0 && col_a + ra <= ldp && col_g + rg <= ldp, "gl3_delta_inner: columns beyond the rows of %d", ldp);
  GL3_REQUIRE(Na % 64 == 0 && Ng % 64 == 0 && Na >= H * D && Ng >= H * Dv && (uintptr_t)w2 % 16 == 0,
              "gl3_delta_inner: %d and %d rows for %d heads of %d and %d", Na, Ng, H, D, Dv);
  const DeltaInner s{ldp, col_a, ra, col_g, rg, Rp, Na, H * D, H * Dv, D, T};
  const unsigned nb = (unsigned)((Na + Ng) / 64);
  if (w_dtype == GL3_F32) {
    GL3_REQUIRE((T + 3) / 4 <= 65535, "gl3_delta_inner: %d tokens exceed the grid", T);
    delta_inner_f32_kernel<<<dim3(nb, (T + 3) / 4), dim3(256), 0, stream>>>(proj, (const float*)w2, A_log, dt_bias, decay, gate, s);
  } else if (w_dtype == GL3_BF16) {
    const int mt = T <= 16 ? 1 : 4;
    const size_t lds = (size_t)16 * mt * (Rp + 8) * sizeof(bf16_t);
    GL3_REQUIRE((T + 16 * mt - 1) / (16 * mt) <= 65535 && (lds <= 64 * 1024 || mt > 1), "gl3_delta_inner: %d tokens of %d", T, Rp);
    if (mt == 1 || lds > 64 * 1024)
      delta_inner_mfma_kernel<1><<<dim3(nb, (T + 15) / 16), dim3(256), (size_t)16 * (Rp + 8) * sizeof(bf16_t), stream>>>(
          proj, (const bf16_t*)w2, A_log, dt_bias, decay, gate, s);
    else
      delta_inner_mfma_kernel<4><<<dim3(nb, (T + 63) / 64), dim3(256), lds, stream>>>(proj, (const bf16_t*)w2, A_log, dt_bias,
                                                                                      decay, gate, s);
  } else {
    GL3_REQUIRE(false, "gl3_delta_inner: unknown dtype %d", w_dtype);
  }
  GL3_LAUNCH_CHECK();
  return 0;
}
