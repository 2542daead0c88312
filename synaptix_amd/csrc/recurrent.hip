// Mixers that carry a state of fixed size from token to token, and the short causal convolution in front of them.
//
//   short_conv         y_t[c] = act(bias[c] + sum_j w[c][j] u_(t - taps + 1 + j)[c]) over each sequence's own tokens; the
//                      last taps - 1 inputs of a sequence are kept in its state row, so a step goes on where the last
//                      one stopped (zeros before a sequence's first token: a fresh state row is zero)
//   state_space_scan   a scalar decay a head:   S <- exp(-exp(A) dt) S + dt B x^T,  y = S^T C + D x      (S: N x P)
//   channel_delta_scan a decay for every key channel and the delta rule:
//                      S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q                 (S: D x P)
//   head_delta_scan    the same with one decay a head, S <- g S (prompts in chunks on the matrix cores)
//   gated_linear_scan  a decay for every key channel, no correction: S <- diag(g) S + k v^T,  o = S^T q   (S: D x P; prompts in
//                      chunks on the matrix cores), gated_linear_step: single tokens, with the heads' norm and gate
//   diff_heads         two softmax maps over the same values, o = rms_norm(a1 - lambda a2) (1 - c)
//
// Everything here is 32-bit FMA: inputs are the float sums of the projections, states are float.  The scans walk a
// sequence's tokens in order; what runs side by side is (sequence, head, columns of the state): a wave holds some columns
// of a head's state in registers, several lanes a column, each with its share of the rows.  A workgroup's waves (64
// columns of one head) share the token's vectors, which are staged through LDS up to 32 tokens at a time; the next
// tokens' vectors are asked for from memory before this chunk's tokens are walked.
#include "common.h"

#define RC_MAX_TAPS 16
#define RC_TB 32            // the most tokens staged at a time (fewer where LDS would not hold them)
#define RC_ROWS_MAX 256     // rows of a head's state (N of the state space, key size of the delta rule)

__device__ __forceinline__ float rc_silu(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float rc_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ---------------------------------------------------------------- short causal convolution
// u: float rows of u_stride values (columns of a fused projection); state [rows][taps - 1][C]; out [N][C].
// One thread a (token, channel).  A sequence's tokens lie one after another, so the input `back` tokens earlier is
// `back` rows up, or, before the step's first token, in the state.
__global__ void __launch_bounds__(256)
short_conv_kernel(const float* __restrict__ u, int u_stride, const float* __restrict__ w, const float* __restrict__ bias,
                  int act, const float* __restrict__ state, int state_rows, const int* __restrict__ tok_seq,
                  const int* __restrict__ tok_pos, const int* __restrict__ seq_past, const int* __restrict__ seq_slot,
                  float* __restrict__ out, int N, int C, int taps) {
  const int c = blockIdx.y * blockDim.x + threadIdx.x, n = blockIdx.x;     // (tokens along x: any number of them)
  if (c >= C) return;
  const int seq = tok_seq[n], in_step = tok_pos[n] - seq_past[seq];       // new tokens of the sequence before this one
  int slot = seq_slot[seq];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const float* st = state + (size_t)slot * (taps - 1) * C;
  float acc = bias ? bias[c] : 0.f;
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;
    const float v = back <= in_step ? u[(size_t)(n - back) * u_stride + c] : st[(size_t)(taps - 1 - (back - in_step)) * C + c];
    acc = fmaf(w[(size_t)c * taps + j], v, acc);
  }
  out[(size_t)n * C + c] = act ? rc_silu(acc) : acc;
}

// The state after the step: the last taps - 1 inputs of (old state, the step's inputs).  One thread a (sequence,
// channel) reads what it keeps before it writes.
__global__ void __launch_bounds__(256)
short_conv_state_kernel(const float* __restrict__ u, int u_stride, float* __restrict__ state, int state_rows,
                        const int* __restrict__ seq_start, const int* __restrict__ seq_slot, int C, int taps) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x, b = blockIdx.y;
  if (c >= C) return;
  int slot = seq_slot[b];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const int s0 = seq_start[b], n_new = seq_start[b + 1] - s0, keep = taps - 1;
  float* st = state + (size_t)slot * keep * C;
  float v[RC_MAX_TAPS];
#pragma unroll
  for (int i = 0; i < RC_MAX_TAPS; ++i) {
    if (i < keep) {
      const int from_end = keep - i;            // the value that ends up in place i is this many inputs from the end
      v[i] = from_end <= n_new ? u[(size_t)(s0 + n_new - from_end) * u_stride + c] : st[(size_t)(i + n_new) * C + c];
    }
  }
#pragma unroll
  for (int i = 0; i < RC_MAX_TAPS; ++i)
    if (i < keep) st[(size_t)i * C + c] = v[i];
}

// Single tokens (every sequence of the step brings one): output and the state's shift in one pass, one thread a
// (sequence, channel), which reads what it needs before it writes.
__global__ void __launch_bounds__(256)
short_conv_single_kernel(const float* __restrict__ u, int u_stride, const float* __restrict__ w, const float* __restrict__ bias,
                         int act, float* __restrict__ state, int state_rows, const int* __restrict__ seq_start,
                         const int* __restrict__ seq_slot, float* __restrict__ out, int C, int taps) {
  const int c = blockIdx.y * blockDim.x + threadIdx.x, b = blockIdx.x;
  if (c >= C) return;
  int slot = seq_slot[b];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const int n = seq_start[b], keep = taps - 1;
  float* st = state + (size_t)slot * keep * C;
  const float now = u[(size_t)n * u_stride + c];
  float v[RC_MAX_TAPS];
  float acc = bias ? bias[c] : 0.f;
#pragma unroll
  for (int i = 0; i < RC_MAX_TAPS; ++i)
    if (i < keep) {
      v[i] = st[(size_t)i * C + c];
      acc = fmaf(w[(size_t)c * taps + i], v[i], acc);
    }
  acc = fmaf(w[(size_t)c * taps + keep], now, acc);
  out[(size_t)n * C + c] = act ? rc_silu(acc) : acc;
#pragma unroll
  for (int i = 0; i < RC_MAX_TAPS; ++i)
    if (i < keep) st[(size_t)i * C + c] = i + 1 < keep ? v[i + 1 < RC_MAX_TAPS ? i + 1 : i] : now;
}

SYN_EXPORT int syn_short_conv(const float* u, int u_stride, const float* w, const float* bias, int act, float* state,
                              int state_rows, const int* tok_seq, const int* tok_pos, const int* seq_start,
                              const int* seq_past, const int* seq_slot, float* out, int n_tokens, int n_seqs, int C,
                              int taps, hipStream_t stream) {
  SYN_CHECK(n_tokens > 0 && n_seqs > 0 && C > 0, "short_conv: empty input");
  SYN_CHECK(taps >= 1 && taps <= RC_MAX_TAPS, "short_conv: %d taps (1 to %d)", taps, RC_MAX_TAPS);
  SYN_CHECK(u_stride >= C && state_rows > 0, "short_conv: rows of %d values for %d channels", u_stride, C);
  const int bx = (C + 255) / 256;
  if (n_tokens == n_seqs) {      // (a step brings at least one token for each of its sequences: here exactly one)
    short_conv_single_kernel<<<dim3(n_seqs, bx), 256, 0, stream>>>(u, u_stride, w, bias, act, state, state_rows, seq_start,
                                                                  seq_slot, out, C, taps);
    SYN_LAUNCH_CHECK("short_conv_single");
    return 0;
  }
  short_conv_kernel<<<dim3(n_tokens, bx), 256, 0, stream>>>(u, u_stride, w, bias, act, state, state_rows, tok_seq, tok_pos,
                                                           seq_past, seq_slot, out, n_tokens, C, taps);
  SYN_LAUNCH_CHECK("short_conv");
  if (taps > 1) {
    short_conv_state_kernel<<<dim3(bx, n_seqs), 256, 0, stream>>>(u, u_stride, state, state_rows, seq_start, seq_slot, C, taps);
    SYN_LAUNCH_CHECK("short_conv_state");
  }
  return 0;
}

// ---------------------------------------------------------------- what the two scans share
// A wave holds 64 / SL columns of a head's state, SL lanes a column (SL = 4 or 16 slices), and a lane holds the rows
// slice * R .. slice * R + R - 1 of its column (R = rows / SL rounded up to a multiple of 4; rows beyond the state's are
// zeros that stay zeros).
//   SL = 4:  lane = 16 * slice + column.  The state is read and written in pieces of 64 bytes: for single tokens, where
//            the state is all that moves.
//   SL = 16: lane = slice + 16 * column.  A token's chain of operations is a quarter as long, there are four times as many
//            waves, and the sum over a column's slices stays inside a row of 16 lanes (four DPP additions, no trip through
//            LDS): for prompts, whose tokens come one after another and wait for one another.
// A token's vectors over the rows lie in LDS as SL pieces of R values, each followed by four unused ones, so that the
// slices' 16-byte reads spread over the banks and no read needs a bound.
#define RC_LD(R, SL) ((SL) * ((R) + 4))
#define RC_LDS_BUDGET (60 * 1024)
#define RC_PF(R) ((R) <= 8 ? 8 : 4)   // row values (each of two vectors) that a thread of the state space's scan holds of the next chunk
#define RC_PFX 2     // column values likewise
#define RC_TPW 2     // tokens that a wave of the delta rule's scan holds of the next chunk
__device__ __forceinline__ int rc_at(int n, int R) { return (n / R) * (R + 4) + n % R; }
template <int CTRL>
__device__ __forceinline__ float rc_dpp(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
// the sum over the lanes that hold a column's slices, in all of them
template <int SL>
__device__ __forceinline__ float rc_sum_slices(float v) {
  if constexpr (SL == 16) {
    v += rc_dpp<0xB1>(v);       // lanes 1 0 3 2 of every four
    v += rc_dpp<0x4E>(v);       // lanes 2 3 0 1
    v += rc_dpp<0x141>(v);      // the other four of every eight (mirrored)
    v += rc_dpp<0x140>(v);      // the other eight of the row (mirrored)
  } else {
#pragma unroll
    for (int off = 64 / SL; off < SYN_WAVE; off <<= 1) v += __shfl_xor(v, off, SYN_WAVE);
  }
  return v;
}
template <int SL> __device__ __forceinline__ int rc_slice(int lane) { return SL == 16 ? lane % 16 : lane / (64 / SL); }
template <int SL> __device__ __forceinline__ int rc_col(int lane) { return SL == 16 ? lane / 16 : lane % (64 / SL); }

// How many of a head's columns a workgroup takes (64, 32 or 16): a token's work for one head is bounded by what one
// compute unit issues, so a prompt's heads are spread over as many compute units as there are (their workgroups then
// stage the same row vectors each for itself); single tokens keep 64.
static int rc_block_columns(long heads, int cols, int longest) {
  if (longest <= 1) return 64;
  const long units = syn_compute_units();
  for (int cb = 64; cb > 16; cb /= 2)
    if (heads * ((cols + cb - 1) / cb) >= units) return cb;
  return 16;
}
// Four slices a wave (a lane then does four times the rows for the same overhead a token) also for prompts, where the
// chip has two waves a SIMD even so.
static bool rc_few_slices(long heads, int cols) { return heads * ((cols + 15) / 16) >= 8L * syn_compute_units(); }

// ---------------------------------------------------------------- state space with a scalar decay a head
// xbc [N][inner + 2 G Ns] float: x (H x P), B (G x Ns), C (G x Ns) behind the convolution; dt: float rows of dt_stride
// values, one a head, before bias and softplus; state [rows][H][Ns][P]; y [N][H * P] float (D x included).
template <int R, int SL>
__global__ void __launch_bounds__(64 * SL)
state_space_scan_kernel(const float* __restrict__ xbc, const float* __restrict__ dt, int dt_stride,
                        const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ d_skip,
                        float* __restrict__ state, int state_rows, const int* __restrict__ seq_start,
                        const int* __restrict__ seq_slot, float* __restrict__ y, int H, int P, int Ns, int G, int tb_max) {
  constexpr int LD = RC_LD(R, SL), COLS = 64 / SL;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* Bs = lds;                          // [tb_max][LD]
  float* Cs = Bs + tb_max * LD;             // [tb_max][LD]
  float* xs = Cs + tb_max * LD;             // [tb_max][64]   dt * x of the workgroup's columns
  float* xr = xs + tb_max * 64;             // [tb_max][64]   x itself
  float* dec = xr + tb_max * 64;            // [tb_max]
  const int CB = blockDim.x / SYN_WAVE * (64 / SL);      // columns of this workgroup
  const int head = blockIdx.x, b = blockIdx.y, p0 = blockIdx.z * CB;
  const int tid = threadIdx.x, wave = tid / SYN_WAVE, lane = tid % SYN_WAVE, slice = rc_slice<SL>(lane);
  const int mine = wave * COLS + rc_col<SL>(lane), p = p0 + mine;       // this lane's column: of the workgroup's 64, of the head
  const bool col_ok = p < P;
  const int s0 = seq_start[b], n_new = seq_start[b + 1] - s0;
  int slot = seq_slot[b];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const int inner = H * P, width = inner + 2 * G * Ns, grp = head / (H / G);
  float* S = state + ((size_t)slot * H + head) * Ns * P;
  float s[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int n = slice * R + i;
    s[i] = (col_ok && n < Ns) ? S[(size_t)n * P + p] : 0.f;
  }
  const float A = -expf(a_log[head]), bias = dt_bias[head], D = d_skip[head];
  // a chunk's values on their way from memory: asked for while the chunk before is walked (the host keeps a chunk within
  // RC_PF(R) row values and RC_PFX column values a thread)
  float pb[RC_PF(R)], pc[RC_PF(R)], px[RC_PFX], pd[RC_PFX];
  auto fetch = [&](int t0) {
    const int tb = min(tb_max, n_new - t0);
#pragma unroll
    for (int j = 0; j < RC_PF(R); ++j) {
      const int e = tid + j * blockDim.x, t = e / (SL * R), n = e % (SL * R);
      pb[j] = pc[j] = 0.f;
      if (e < tb * SL * R && n < Ns) {
        const float* row = xbc + (size_t)(s0 + t0 + t) * width + inner + grp * Ns;
        pb[j] = row[n];
        pc[j] = row[G * Ns + n];
      }
    }
#pragma unroll
    for (int j = 0; j < RC_PFX; ++j) {
      const int e = tid + j * blockDim.x, t = e / CB, pp = p0 + e % CB;
      px[j] = pd[j] = 0.f;
      if (e < tb * CB) {
        const size_t tok = s0 + t0 + t;
        pd[j] = dt[tok * dt_stride + head];
        if (pp < P) px[j] = xbc[tok * width + head * P + pp];
      }
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n_new; t0 += tb_max) {
    const int tb = min(tb_max, n_new - t0);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < RC_PF(R); ++j) {
      const int e = tid + j * blockDim.x, t = e / (SL * R), n = e % (SL * R);
      if (e < tb * SL * R) {
        Bs[t * LD + rc_at(n, R)] = pb[j];
        Cs[t * LD + rc_at(n, R)] = pc[j];
      }
    }
#pragma unroll
    for (int j = 0; j < RC_PFX; ++j) {
      const int e = tid + j * blockDim.x;
      if (e < tb * CB) {
        const float step = rc_softplus(pd[j] + bias);
        const int at = (e / CB) * 64 + e % CB;
        xs[at] = step * px[j];
        xr[at] = px[j];
        if (e % CB == 0) dec[e / CB] = expf(A * step);
      }
    }
    __syncthreads();
    if (t0 + tb_max < n_new) fetch(t0 + tb_max);
#pragma unroll 2
    for (int t = 0; t < tb; ++t) {
      const float a = dec[t], bx = xs[t * 64 + mine];
      const float4* Bt = (const float4*)(Bs + t * LD + slice * (R + 4));
      const float4* Ct = (const float4*)(Cs + t * LD + slice * (R + 4));
      float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < R; i += 4) {
        const float4 bv = Bt[i / 4], cv = Ct[i / 4];
        s[i] = fmaf(a, s[i], bx * bv.x), acc[0] = fmaf(s[i], cv.x, acc[0]);
        s[i + 1] = fmaf(a, s[i + 1], bx * bv.y), acc[1] = fmaf(s[i + 1], cv.y, acc[1]);
        s[i + 2] = fmaf(a, s[i + 2], bx * bv.z), acc[2] = fmaf(s[i + 2], cv.z, acc[2]);
        s[i + 3] = fmaf(a, s[i + 3], bx * bv.w), acc[3] = fmaf(s[i + 3], cv.w, acc[3]);
      }
      const float sum = rc_sum_slices<SL>((acc[0] + acc[1]) + (acc[2] + acc[3]));
      if (slice == 0 && col_ok)
        y[(size_t)(s0 + t0 + t) * inner + head * P + p] = fmaf(D, xr[t * 64 + mine], sum);
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int n = slice * R + i;
    if (col_ok && n < Ns) S[(size_t)n * P + p] = s[i];
  }
}

SYN_EXPORT int syn_state_space_scan(const float* xbc, const float* dt, int dt_stride, const float* dt_bias,
                                    const float* a_log, const float* d_skip, float* state, int state_rows,
                                    const int* seq_start, const int* seq_slot, int n_seqs, int longest, float* y, int H,
                                    int P, int Ns, int G, hipStream_t stream) {
  SYN_CHECK(n_seqs > 0 && longest > 0 && H > 0 && P > 0 && Ns > 0 && G > 0, "state_space_scan: empty input");
  SYN_CHECK(H % G == 0, "state_space_scan: %d heads do not divide into %d groups", H, G);
  SYN_CHECK(Ns <= RC_ROWS_MAX, "state_space_scan: a state of %d rows (at most %d)", Ns, RC_ROWS_MAX);
  SYN_CHECK(dt_stride >= H && state_rows > 0, "state_space_scan: step rows of %d values for %d heads", dt_stride, H);
  const int block_cols = rc_block_columns((long)H * n_seqs, P, longest);
  // single tokens: four slices a wave (the state moves in pieces of 64 bytes); tokens in a row: sixteen
#define SYN_SS(R, SL)                                                                                                   \
  do {                                                                                                                  \
    const int per_token = (2 * RC_LD(R, SL) + 2 * 64 + 1) * (int)sizeof(float);                                         \
    const int waves = (min(P, block_cols) + 64 / SL - 1) / (64 / SL), cb = waves * (64 / SL);                           \
    const dim3 grid(H, n_seqs, (P + cb - 1) / cb);                                                                      \
    int tb = min(min(RC_TB, longest), RC_LDS_BUDGET / per_token);                                                       \
    tb = max(1, min(tb, min(RC_PF(R) * waves * SYN_WAVE / (SL * R), RC_PFX * waves * SYN_WAVE / cb)));                  \
    state_space_scan_kernel<R, SL><<<grid, waves * SYN_WAVE, (size_t)tb * per_token, stream>>>(                         \
        xbc, dt, dt_stride, dt_bias, a_log, d_skip, state, state_rows, seq_start, seq_slot, y, H, P, Ns, G, tb);        \
  } while (0)
  if (longest <= 1 || rc_few_slices((long)H * n_seqs, P)) {
    if (Ns <= 32) SYN_SS(8, 4);
    else if (Ns <= 64) SYN_SS(16, 4);
    else if (Ns <= 128) SYN_SS(32, 4);
    else SYN_SS(64, 4);
  } else {
    if (Ns <= 64) SYN_SS(4, 16);
    else if (Ns <= 128) SYN_SS(8, 16);
    else SYN_SS(16, 16);
  }
#undef SYN_SS
  SYN_LAUNCH_CHECK("state_space_scan");
  return 0;
}

// ---------------------------------------------------------------- delta rule, a decay for every key channel or one a head
// qkv [N][(2 K + H E)] float behind the convolution: q (K heads x D), k (K x D), v (H x E); beta: float rows, one a head,
// before the sigmoid; a: float rows of a_stride values, before bias and softplus, of which H * D are used (CHANNEL: a decay
// for every key channel) or H (one a head); state [rows][H][D][E]; o [N][H * E] float.
// Staged for each token: q and k as unit vectors (q also times q_scale), the decays, k . q.
template <int R, int SL, bool CHANNEL>
__global__ void __launch_bounds__(64 * SL)
delta_scan_kernel(const float* __restrict__ qkv, const float* __restrict__ beta, int beta_stride,
                          const float* __restrict__ a, int a_stride, const float* __restrict__ a_bias,
                          const float* __restrict__ a_log, float q_scale, float unit_eps, float* __restrict__ state,
                          int state_rows, const int* __restrict__ seq_start, const int* __restrict__ seq_slot,
                          float* __restrict__ o, int H, int K, int D, int E, int tb_max) {
  constexpr int LD = RC_LD(R, SL), COLS = 64 / SL;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* qs = lds;                          // [tb_max][LD]
  float* ks = qs + tb_max * LD;             // [tb_max][LD]
  float* gs = ks + tb_max * LD;             // [tb_max][LD], or [tb_max] with one decay a head
  float* vs = gs + tb_max * (CHANNEL ? LD : 1);      // [tb_max][64]
  float* kq = vs + tb_max * 64;             // [tb_max]
  float* bt = kq + tb_max;                  // [tb_max]
  const int CB = blockDim.x / SYN_WAVE * (64 / SL);      // columns of this workgroup
  const int head = blockIdx.x, b = blockIdx.y, p0 = blockIdx.z * CB;
  const int tid = threadIdx.x, wave = tid / SYN_WAVE, lane = tid % SYN_WAVE, slice = rc_slice<SL>(lane);
  const int n_waves = blockDim.x / SYN_WAVE;
  const int mine = wave * COLS + rc_col<SL>(lane), p = p0 + mine;
  const bool col_ok = p < E;
  const int s0 = seq_start[b], n_new = seq_start[b + 1] - s0;
  int slot = seq_slot[b];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const int kvh = head / (H / K), width = 2 * K * D + H * E;
  float* S = state + ((size_t)slot * H + head) * D * E;
  float s[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int n = slice * R + i;
    s[i] = (col_ok && n < D) ? S[(size_t)n * E + p] : 0.f;
  }
  const float A = -expf(a_log[head]);
  // a chunk's values on their way from memory: a wave stages the tokens wave, wave + n_waves (the host keeps a chunk within
  // RC_TPW tokens a wave), asked for while the chunk before is walked
  constexpr int DL = (SL * R + 63) / 64;
  constexpr int AL = CHANNEL ? DL : 1;
  float pq[RC_TPW][DL], pk[RC_TPW][DL], pa[RC_TPW][AL], pv[RC_TPW], pbeta[RC_TPW];
  auto fetch = [&](int t0) {
    const int tb = min(tb_max, n_new - t0);
#pragma unroll
    for (int j = 0; j < RC_TPW; ++j) {
      const int t = wave + j * n_waves;
      pv[j] = pbeta[j] = 0.f;
#pragma unroll
      for (int i = 0; i < DL; ++i) pq[j][i] = pk[j][i] = 0.f;
#pragma unroll
      for (int i = 0; i < AL; ++i) pa[j][i] = 0.f;
      if (t < tb) {
        const size_t tok = s0 + t0 + t;
        const float* qr = qkv + tok * width + kvh * D;
        const float* kr = qr + K * D;
#pragma unroll
        for (int i = 0; i < DL; ++i) {
          const int d = lane + 64 * i;
          if (d < D) {
            pq[j][i] = qr[d], pk[j][i] = kr[d];
            if constexpr (CHANNEL) pa[j][i] = a[tok * (size_t)a_stride + head * D + d] + a_bias[head * D + d];
          }
        }
        if constexpr (!CHANNEL) pa[j][0] = a[tok * (size_t)a_stride + head] + a_bias[head];
        if (lane < CB && p0 + lane < E) pv[j] = qkv[tok * width + 2 * K * D + head * E + p0 + lane];
        pbeta[j] = beta[tok * beta_stride + head];
      }
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n_new; t0 += tb_max) {
    const int tb = min(tb_max, n_new - t0);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < RC_TPW; ++j) {
      const int t = wave + j * n_waves;
      if (t < tb) {
        float sq = 0.f, sk = 0.f, dot = 0.f;
#pragma unroll
        for (int i = 0; i < DL; ++i)
          sq = fmaf(pq[j][i], pq[j][i], sq), sk = fmaf(pk[j][i], pk[j][i], sk), dot = fmaf(pq[j][i], pk[j][i], dot);
        sq = wave_sum(sq), sk = wave_sum(sk), dot = wave_sum(dot);
        const float iq = q_scale / sqrtf(sq + unit_eps), ik = 1.f / sqrtf(sk + unit_eps);
#pragma unroll
        for (int i = 0; i < DL; ++i) {      // (rows beyond the keys: zeros, and a decay of one)
          const int d = lane + 64 * i;
          if (d < SL * R) {
            const int at = t * LD + rc_at(d, R);
            qs[at] = pq[j][i] * iq;
            ks[at] = pk[j][i] * ik;
            if constexpr (CHANNEL) gs[at] = d < D ? expf(A * rc_softplus(pa[j][i])) : 1.f;
          }
        }
        if (lane == 0) {
          if constexpr (!CHANNEL) gs[t] = expf(A * rc_softplus(pa[j][0]));
          kq[t] = dot * iq * ik;
          bt[t] = 1.f / (1.f + expf(-pbeta[j]));
        }
        vs[t * 64 + lane] = pv[j];
      }
    }
    __syncthreads();
    if (t0 + tb_max < n_new) fetch(t0 + tb_max);
#pragma unroll 1
    for (int t = 0; t < tb; ++t) {
      const float4* qt = (const float4*)(qs + t * LD + slice * (R + 4));
      const float4* kt = (const float4*)(ks + t * LD + slice * (R + 4));
      float rk[4] = {0.f, 0.f, 0.f, 0.f}, rq[4] = {0.f, 0.f, 0.f, 0.f};
      if constexpr (CHANNEL) {
        const float4* gt = (const float4*)(gs + t * LD + slice * (R + 4));
#pragma unroll
        for (int i = 0; i < R; i += 4) {
          const float4 gv = gt[i / 4], kv = kt[i / 4], qv = qt[i / 4];
          s[i] *= gv.x, rk[0] = fmaf(s[i], kv.x, rk[0]), rq[0] = fmaf(s[i], qv.x, rq[0]);
          s[i + 1] *= gv.y, rk[1] = fmaf(s[i + 1], kv.y, rk[1]), rq[1] = fmaf(s[i + 1], qv.y, rq[1]);
          s[i + 2] *= gv.z, rk[2] = fmaf(s[i + 2], kv.z, rk[2]), rq[2] = fmaf(s[i + 2], qv.z, rq[2]);
          s[i + 3] *= gv.w, rk[3] = fmaf(s[i + 3], kv.w, rk[3]), rq[3] = fmaf(s[i + 3], qv.w, rq[3]);
        }
      } else {
        // one decay for the whole state: it multiplies the sums over the old state instead, (g S)^T k = g (S^T k)
#pragma unroll
        for (int i = 0; i < R; i += 4) {
          const float4 kv = kt[i / 4], qv = qt[i / 4];
          rk[0] = fmaf(s[i], kv.x, rk[0]), rq[0] = fmaf(s[i], qv.x, rq[0]);
          rk[1] = fmaf(s[i + 1], kv.y, rk[1]), rq[1] = fmaf(s[i + 1], qv.y, rq[1]);
          rk[2] = fmaf(s[i + 2], kv.z, rk[2]), rq[2] = fmaf(s[i + 2], qv.z, rq[2]);
          rk[3] = fmaf(s[i + 3], kv.w, rk[3]), rq[3] = fmaf(s[i + 3], qv.w, rq[3]);
        }
      }
      float rks = rc_sum_slices<SL>((rk[0] + rk[1]) + (rk[2] + rk[3]));
      float rqs = rc_sum_slices<SL>((rq[0] + rq[1]) + (rq[2] + rq[3]));
      float g = 1.f;
      if constexpr (!CHANNEL) g = gs[t], rks *= g, rqs *= g;
      const float u = bt[t] * (vs[t * 64 + mine] - rks);
#pragma unroll
      for (int i = 0; i < R; i += 4) {
        const float4 kv = kt[i / 4];
        if constexpr (CHANNEL) {
          s[i] = fmaf(kv.x, u, s[i]), s[i + 1] = fmaf(kv.y, u, s[i + 1]);
          s[i + 2] = fmaf(kv.z, u, s[i + 2]), s[i + 3] = fmaf(kv.w, u, s[i + 3]);
        } else {
          s[i] = fmaf(kv.x, u, g * s[i]), s[i + 1] = fmaf(kv.y, u, g * s[i + 1]);
          s[i + 2] = fmaf(kv.z, u, g * s[i + 2]), s[i + 3] = fmaf(kv.w, u, g * s[i + 3]);
        }
      }
      // the read-out sees this token's write: (S + k u^T)^T q = S^T q + u (k . q)
      if (slice == 0 && col_ok) o[(size_t)(s0 + t0 + t) * H * E + head * E + p] = fmaf(u, kq[t], rqs);
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int n = slice * R + i;
    if (col_ok && n < D) S[(size_t)n * E + p] = s[i];
  }
}

// ---------------------------------------------------------------- delta rule with one decay a head, prompts in chunks
// With a decay for the whole state a chunk of C tokens is a few small products.  From the state S before the chunk, with
// G_t = g_1 .. g_t and G_tj = g_(j+1) .. g_t (products of at most C decays, no quotient):
//   u_t = b_t (v_t - G_t S^T k_t - sum_(j<t) G_tj (k_t . k_j) u_j)        so  (I + L) U = diag(b) (V - diag(G) K S)
//   o_t = G_t S^T q_t + sum_(j<=t) G_tj (q_t . k_j) u_j                      with L_tj = b_t G_tj (k_t . k_j), j < t
//   S'  = G_C S + sum_j G_Cj k_j u_j^T
// (the unrolled recurrence; the triangular system of the delta rule's chunked form: S. Yang, B. Wang, Y. Zhang, Y. Shen,
// Y. Kim, "Parallelizing Linear Transformers with the Delta Rule over Sequence Length").  T = (I + L)^-1 diag(b),
// A_tj = G_tj (q_t . k_j) and the decays do not depend on the state: head_delta_chunks_kernel makes them for all chunks side by
// side.  head_delta_carry_kernel then walks the chunks:  U = T (V - diag(G) K S),  O = diag(G) Q S + A U,
// S <- G_C S + K^T diag(G_Cj) U, on the matrix cores in 32-bit (16x16x4).
//
// C = 16 is that instruction's side.  Everything lies in the order of its operands: a wave holds 16 columns of a head's
// state as accumulators (lane = 16 g + n has rows 16 i + 4 g + j of column n), and an accumulator is also the B operand of the
// next product if the k index of step j counts the rows 4 g + j, so neither the state nor U ever moves between lanes.  The
// A operands of four steps are then four consecutive values of a row: "fragments" [tile][lane][4] of 1 KB.
#define HDC 16
typedef f32x4 hd_frag;

// floats of one (chunk, key head): K, Q and K^T in fragments; of one (chunk, head): T, A, [G_t], [G_Cj]
__host__ __device__ __forceinline__ size_t hd_key_floats(int NT) { return (size_t)3 * NT * 256; }
#define HD_HEAD_FLOATS (2 * 256 + 2 * HDC)

// Which sequence and chunk a place of the chunk arrays is: sequence b's chunks begin at seq_start[b] / C + b, which leaves
// room for every sequence's last, partly filled chunk.  False for places of no chunk.
__device__ __forceinline__ bool hd_chunk_of(int place, const int* __restrict__ seq_start, int n_seqs, int& first, int& n) {
  for (int b = 0; b < n_seqs; ++b) {
    const int s0 = seq_start[b], s1 = seq_start[b + 1], at = place - (s0 / HDC + b);
    if (at >= 0 && at * HDC < s1 - s0) {
      first = s0 + at * HDC, n = min(HDC, s1 - first);
      return true;
    }
  }
  return false;
}

// One workgroup a (chunk, key head), and the heads that read it.
__global__ void __launch_bounds__(256)
head_delta_chunks_kernel(const float* __restrict__ qkv, const float* __restrict__ beta, int beta_stride,
                         const float* __restrict__ a, int a_stride, const float* __restrict__ a_bias,
                         const float* __restrict__ a_log, float q_scale, float unit_eps, const int* __restrict__ seq_start,
                         int n_seqs, float* __restrict__ keys, float* __restrict__ heads, int H, int K, int D, int E, int NT) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int LDD = 16 * NT + 1;
  float* ks = lds;                        // [C][LDD] unit keys, zeros beyond the keys and the chunk's tokens
  float* qs = ks + HDC * LDD;             // [C][LDD] unit queries times q_scale
  float* kk = qs + HDC * LDD;             // [C][C + 1] k_t . k_j
  float* qk = kk + HDC * (HDC + 1);       // [C][C + 1] q_t . k_j
  float* Ls = qk + HDC * (HDC + 1);       // [4 waves][C][C + 1]
  float* gs = Ls + 4 * HDC * (HDC + 1);   // [4 waves][2][C] decays, steps
  int first, n;
  if (!hd_chunk_of(blockIdx.x, seq_start, n_seqs, first, n)) return;      // (the whole workgroup)
  const int kvh = blockIdx.y, tid = threadIdx.x, wave = tid / SYN_WAVE, lane = tid % SYN_WAVE;
  const int width = 2 * K * D + H * E;
  for (int t = wave; t < HDC; t += 4) {
    const float* qr = qkv + (size_t)(first + min(t, n - 1)) * width + kvh * D;
    const float* kr = qr + K * D;
    float q[RC_ROWS_MAX / SYN_WAVE], k[RC_ROWS_MAX / SYN_WAVE], sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < RC_ROWS_MAX / SYN_WAVE; ++i) {
      const int d = lane + i * SYN_WAVE;
      const bool in = t < n && d < D;
      q[i] = in ? qr[d] : 0.f, k[i] = in ? kr[d] : 0.f;
      sq = fmaf(q[i], q[i], sq), sk = fmaf(k[i], k[i], sk);
    }
    sq = wave_sum(sq), sk = wave_sum(sk);
    const float iq = q_scale / sqrtf(sq + unit_eps), ik = 1.f / sqrtf(sk + unit_eps);
#pragma unroll
    for (int i = 0; i < RC_ROWS_MAX / SYN_WAVE; ++i) {
      const int d = lane + i * SYN_WAVE;
      if (d < 16 * NT) qs[t * LDD + d] = q[i] * iq, ks[t * LDD + d] = k[i] * ik;
    }
  }
  __syncthreads();
  // the fragments of K (row m = token, k = 4 g + j), Q and K^T (row m = key value, k = token 4 g + j)
  float* kf = keys + ((size_t)blockIdx.x * K + kvh) * hd_key_floats(NT);
  for (int e = tid; e < NT * 64; e += 256) {
    const int tile = e / 64, m = e % 16, g = (e % 64) / 16;
    hd_frag fk, fq, ft;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      fk[j] = ks[m * LDD + 16 * tile + 4 * g + j];
      fq[j] = qs[m * LDD + 16 * tile + 4 * g + j];
      ft[j] = ks[(4 * g + j) * LDD + 16 * tile + m];
    }
    ((hd_frag*)kf)[e] = fk, ((hd_frag*)kf)[NT * 64 + e] = fq, ((hd_frag*)kf)[2 * NT * 64 + e] = ft;
  }
  {
    const int t = tid / HDC, j = tid % HDC;
    float dk = 0.f, dq = 0.f;
    for (int d = 0; d < D; ++d) {
      const float kj = ks[j * LDD + d];
      dk = fmaf(ks[t * LDD + d], kj, dk), dq = fmaf(qs[t * LDD + d], kj, dq);
    }
    kk[t * (HDC + 1) + j] = dk, qk[t * (HDC + 1) + j] = dq;
  }
  __syncthreads();
  // a wave a head; what its lanes exchange through LDS is the wave's own (every wave takes the same number of turns, so
  // the barriers are the workgroup's)
  const int rep = H / K;
  float* L = Ls + wave * HDC * (HDC + 1);
  float* gd = gs + wave * 2 * HDC;
  for (int r0 = 0; r0 < rep; r0 += 4) {
    const bool on = r0 + wave < rep;
    const int head = kvh * rep + min(r0 + wave, rep - 1);
    if (lane < HDC) {       // tokens beyond the chunk's: nothing decays, nothing is written
      const size_t tok = first + min(lane, n - 1);
      gd[lane] = lane < n ? expf(-expf(a_log[head]) * rc_softplus(a[tok * a_stride + head] + a_bias[head])) : 1.f;
      gd[HDC + lane] = lane < n ? 1.f / (1.f + expf(-beta[tok * beta_stride + head])) : 0.f;
    }
    __syncthreads();
    float* hf = heads + ((size_t)blockIdx.x * H + head) * HD_HEAD_FLOATS;
    const int j = lane % HDC;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * (lane / HDC) + i;
      float dec = t >= j ? 1.f : 0.f;
      for (int x = j + 1; x <= t; ++x) dec *= gd[x];
      L[t * (HDC + 1) + j] = t > j ? gd[HDC + t] * dec * kk[t * (HDC + 1) + j] : 0.f;
      if (on) {
        hf[256 + ((j / 4) * 16 + t) * 4 + j % 4] = dec * qk[t * (HDC + 1) + j];       // A, row t, k = j
        if (t == HDC - 1) hf[2 * 256 + HDC + j] = dec;                                 // G_Cj
        if (j == 0) hf[2 * 256 + t] = dec * gd[0];                                     // G_t
      }
    }
    __syncthreads();
    if (lane < HDC) {       // column j of (I + L)^-1, row after row
      float col[HDC];
#pragma unroll
      for (int t = 0; t < HDC; ++t) {
        float v = t == j ? 1.f : 0.f;
#pragma unroll
        for (int x = 0; x < t; ++x) v = fmaf(-L[t * (HDC + 1) + x], col[x], v);
        col[t] = v;
      }
      const float step = gd[HDC + j];
      if (on) {
#pragma unroll
        for (int t = 0; t < HDC; ++t) hf[((j / 4) * 16 + t) * 4 + j % 4] = col[t] * step;      // T, row t, k = j
      }
    }
    __syncthreads();
  }
}

__device__ __forceinline__ f32x4 hd_mfma(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// One chunk's operands in a wave's registers.
template <int TPW, int CG>
struct HdOperands {
  hd_frag k[TPW], q[TPW], kt[TPW], T, A;
  f32x4 gt, gc, v[CG];  // G_t and G_Cj of the tokens 4 g + j, their values in this lane's columns
};

// A workgroup for CG groups of 16 columns of a (sequence, head): two where there are enough workgroups even so, since they
// share the keys' operands.  W waves hold TPW tiles of 16 rows of the state each: what a wave's
// rows give to K S and Q S is summed through LDS (two buffers in turns: one barrier a chunk), then every wave makes U and
// updates its rows; one more wave makes and stores the outputs meanwhile.  The operands are asked for two chunks ahead.
template <int TPW, int W, int CG>
__global__ void __launch_bounds__((W + 1) * SYN_WAVE)
head_delta_carry_kernel(const float* __restrict__ qkv, const float* __restrict__ keys, const float* __restrict__ heads,
                        float* __restrict__ state, int state_rows, const int* __restrict__ seq_start,
                        const int* __restrict__ seq_slot, float* __restrict__ o, int H, int K, int D, int E) {
  constexpr int NT = TPW * W;
  __shared__ __attribute__((aligned(16))) f32x4 part[2][W][2][CG][SYN_WAVE];
  const int head = blockIdx.x, b = blockIdx.z, wave = threadIdx.x / SYN_WAVE, lane = threadIdx.x % SYN_WAVE;
  const bool holds = wave < W;                       // (else the wave of the outputs)
  const int g = lane / 16, col = blockIdx.y * 16 * CG + lane % 16;       // (this lane's columns: col, col + 16)
  const int s0 = seq_start[b], n_new = seq_start[b + 1] - s0;
  if (n_new <= 0) return;                            // (the whole workgroup)
  int slot = seq_slot[b];
  if (slot < 0 || slot >= state_rows) slot = state_rows - 1;
  const int kvh = head / (H / K), width = 2 * K * D + H * E;
  float* Sg = state + ((size_t)slot * H + head) * D * E;
  f32x4 S[CG][TPW];
#pragma unroll
  for (int y = 0; y < CG; ++y)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 16 * (wave * TPW + i) + 4 * g + j, c = col + 16 * y;
        S[y][i][j] = (holds && c < E && d < D) ? Sg[(size_t)d * E + c] : 0.f;
      }
  const int chunk0 = s0 / HDC + b, n_chunks = (n_new + HDC - 1) / HDC;
  const float* vp = qkv + (size_t)s0 * width + 2 * K * D + head * E;
  float* op = o + (size_t)s0 * H * E + head * E + col;
  auto ask = [&](HdOperands<TPW, CG>& x, int c) {
    c = min(c, n_chunks - 1);
    const float* hf = heads + ((size_t)(chunk0 + c) * H + head) * HD_HEAD_FLOATS;
    if (holds) {
      const hd_frag* kf = (const hd_frag*)(keys + ((size_t)(chunk0 + c) * K + kvh) * hd_key_floats(NT)) + wave * TPW * 64 + lane;
#pragma unroll
      for (int i = 0; i < TPW; ++i) x.k[i] = kf[i * 64], x.q[i] = kf[(NT + i) * 64], x.kt[i] = kf[(2 * NT + i) * 64];
      x.gc = ((const f32x4*)(hf + 2 * 256 + HDC))[g];
    } else {
      x.A = ((const hd_frag*)(hf + 256))[lane];
    }
    x.T = ((const hd_frag*)hf)[lane];
    x.gt = ((const f32x4*)(hf + 2 * 256))[g];
#pragma unroll
    for (int y = 0; y < CG; ++y)
#pragma unroll
      for (int j = 0; j < 4; ++j)      // (T has zeros for tokens beyond the last; columns beyond are not stored)
        x.v[y][j] = vp[(size_t)min(c * HDC + 4 * g + j, n_new - 1) * width + min(col + 16 * y, E - 1)];
  };
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  auto step = [&](const HdOperands<TPW, CG>& x, int c, int at) {
    if (holds) {
#pragma unroll
      for (int y = 0; y < CG; ++y) {
        f32x4 ks[2] = {zero, zero}, qs[2] = {zero, zero};
#pragma unroll
        for (int i = 0; i < TPW; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            ks[j & 1] = hd_mfma(x.k[i][j], S[y][i][j], ks[j & 1]);
            qs[j & 1] = hd_mfma(x.q[i][j], S[y][i][j], qs[j & 1]);
          }
        part[at][wave][0][y][lane] = ks[0] + ks[1];
        part[at][wave][1][y][lane] = qs[0] + qs[1];
      }
    }
    __syncthreads();
    f32x4 u[CG];
#pragma unroll
    for (int y = 0; y < CG; ++y) {
      f32x4 sum = part[at][0][0][y][lane];
#pragma unroll
      for (int w = 1; w < W; ++w) sum += part[at][w][0][y][lane];
      const f32x4 r = x.v[y] - x.gt * sum;
      u[y] = zero;
#pragma unroll
      for (int j = 0; j < 4; ++j) u[y] = hd_mfma(x.T[j], r[j], u[y]);
    }
    if (holds) {
      const float whole = __shfl(x.gt[3], 48, SYN_WAVE);        // G_C: the last token's
#pragma unroll
      for (int y = 0; y < CG; ++y) {
        const f32x4 uc = x.gc * u[y];
#pragma unroll
        for (int i = 0; i < TPW; ++i) S[y][i] *= whole;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int i = 0; i < TPW; ++i) S[y][i] = hd_mfma(x.kt[i][j], uc[j], S[y][i]);
      }
    } else {
#pragma unroll
      for (int y = 0; y < CG; ++y) {
        f32x4 out = part[at][0][1][y][lane];
#pragma unroll
        for (int w = 1; w < W; ++w) out += part[at][w][1][y][lane];
        out *= x.gt;
#pragma unroll
        for (int j = 0; j < 4; ++j) out = hd_mfma(x.A[j], u[y][j], out);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int t = c * HDC + 4 * g + j;
          if (t < n_new && col + 16 * y < E) op[(size_t)t * H * E + 16 * y] = out[j];
        }
      }
    }
  };
  HdOperands<TPW, CG> even, odd;
  ask(even, 0), ask(odd, 1);
  for (int c = 0; c < n_chunks; c += 2) {
    step(even, c, 0);
    ask(even, c + 2);
    if (c + 1 < n_chunks) {
      step(odd, c + 1, 1);
      ask(odd, c + 3);
    }
  }
#pragma unroll
  for (int y = 0; y < CG; ++y)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 16 * (wave * TPW + i) + 4 * g + j, c = col + 16 * y;
        if (holds && c < E && d < D) Sg[(size_t)d * E + c] = S[y][i][j];
      }
}

static int hd_tiles(int D) {      // tiles of 16 key values: what the walk is built for
  const int need = (D + 15) / 16;
  for (int nt : {1, 2, 4, 8, 12, 16})
    if (need <= nt) return nt;
  return 0;
}

template <bool CHANNEL>
static int delta_scan(const char* name, const float* qkv, const float* beta, int beta_stride, const float* a, int a_stride,
                      const float* a_bias, const float* a_log, float q_scale, float unit_eps, float* state, int state_rows,
                      const int* seq_start, const int* seq_slot, int n_seqs, int longest, float* o, int H, int K, int D, int E,
                      hipStream_t stream) {
  SYN_CHECK(n_seqs > 0 && longest > 0 && H > 0 && K > 0 && D > 0 && E > 0, "%s: empty input", name);
  SYN_CHECK(H % K == 0, "%s: %d heads do not divide into %d key heads", name, H, K);
  SYN_CHECK(D <= RC_ROWS_MAX, "%s: keys of %d values (at most %d)", name, D, RC_ROWS_MAX);
  SYN_CHECK(beta_stride >= H && state_rows > 0, "%s: rows of %d values for %d heads", name, beta_stride, H);
  SYN_CHECK(a_stride >= (CHANNEL ? H * D : H), "%s: decay rows of %d values for %d heads of %d", name, a_stride, H, D);
  // (always 64 columns a workgroup: staging a token here means norms and decays, which workgroups that split a head's
  // columns would each do again; measured at 32 heads over 2,048 tokens: 1.18 ms with 64 columns, 1.46 ms with 16)
  const int block_cols = 64;
#define SYN_CD(R, SL)                                                                                                   \
  do {                                                                                                                  \
    const int per_token = ((CHANNEL ? 3 : 2) * RC_LD(R, SL) + 64 + (CHANNEL ? 2 : 3)) * (int)sizeof(float);             \
    const int waves = (min(E, block_cols) + 64 / SL - 1) / (64 / SL), cb = waves * (64 / SL);                           \
    const dim3 grid(H, n_seqs, (E + cb - 1) / cb);                                                                      \
    const int tb = max(1, min(min(min(RC_TB, longest), RC_LDS_BUDGET / per_token), RC_TPW * waves));                    \
    delta_scan_kernel<R, SL, CHANNEL><<<grid, waves * SYN_WAVE, (size_t)tb * per_token, stream>>>(                      \
        qkv, beta, beta_stride, a, a_stride, a_bias, a_log, q_scale, unit_eps, state, state_rows, seq_start, seq_slot,  \
        o, H, K, D, E, tb);                                                                                             \
  } while (0)
  if (longest <= 1 || rc_few_slices((long)H * n_seqs, E)) {
    if (D <= 32) SYN_CD(8, 4);
    else if (D <= 64) SYN_CD(16, 4);
    else if (D <= 128) SYN_CD(32, 4);
    else SYN_CD(64, 4);
  } else {
    if (D <= 64) SYN_CD(4, 16);
    else if (D <= 128) SYN_CD(8, 16);
    else SYN_CD(16, 16);
  }
#undef SYN_CD
  SYN_LAUNCH_CHECK(name);
  return 0;
}

SYN_EXPORT int syn_channel_delta_scan(const float* qkv, const float* beta, int beta_stride, const float* a, int a_stride,
                                      const float* a_bias, const float* a_log, float q_scale, float unit_eps, float* state,
                                      int state_rows, const int* seq_start, const int* seq_slot, int n_seqs, int longest,
                                      float* o, int H, int K, int D, int E, hipStream_t stream) {
  return delta_scan<true>("channel_delta_scan", qkv, beta, beta_stride, a, a_stride, a_bias, a_log, q_scale, unit_eps, state,
                          state_rows, seq_start, seq_slot, n_seqs, longest, o, H, K, D, E, stream);
}

// floats of scratch memory of a call over prompts
SYN_EXPORT long syn_head_delta_scratch(int n_tokens, int n_seqs, int H, int K, int D) {
  return ((long)n_tokens / HDC + n_seqs) * (K * (long)hd_key_floats(hd_tiles(D)) + H * (long)HD_HEAD_FLOATS);
}

// scratch == nullptr: token by token in one launch (single tokens); else in chunks
SYN_EXPORT int syn_head_delta_scan(const float* qkv, const float* beta, int beta_stride, const float* a, int a_stride,
                                   const float* a_bias, const float* a_log, float q_scale, float unit_eps, float* state,
                                   int state_rows, const int* seq_start, const int* seq_slot, int n_seqs, int longest,
                                   float* o, int H, int K, int D, int E, int n_tokens, float* scratch, hipStream_t stream) {
  if (scratch == nullptr)
    return delta_scan<false>("head_delta_scan", qkv, beta, beta_stride, a, a_stride, a_bias, a_log, q_scale, unit_eps, state,
                             state_rows, seq_start, seq_slot, n_seqs, longest, o, H, K, D, E, stream);
  SYN_CHECK(n_seqs > 0 && n_tokens > 0 && H > 0 && K > 0 && D > 0 && E > 0, "head_delta_scan: empty input");
  SYN_CHECK(H % K == 0, "head_delta_scan: %d heads do not divide into %d key heads", H, K);
  SYN_CHECK(D <= RC_ROWS_MAX, "head_delta_scan: keys of %d values (at most %d)", D, RC_ROWS_MAX);
  SYN_CHECK(beta_stride >= H && a_stride >= H && state_rows > 0, "head_delta_scan: rows of %d and %d values for %d heads",
            beta_stride, a_stride, H);
  SYN_CHECK((uintptr_t)scratch % 16 == 0, "head_delta_scan: the scratch memory is not aligned");
  const int NT = hd_tiles(D), chunks = n_tokens / HDC + n_seqs;
  float* keys = scratch;
  float* heads = scratch + (size_t)chunks * K * hd_key_floats(NT);
  const size_t bytes = (2 * HDC * (16 * NT + 1) + 6 * HDC * (HDC + 1) + 8 * HDC) * sizeof(float);
  head_delta_chunks_kernel<<<dim3(chunks, K), 256, bytes, stream>>>(qkv, beta, beta_stride, a, a_stride, a_bias, a_log, q_scale,
                                                                    unit_eps, seq_start, n_seqs, keys, heads, H, K, D, E, NT);
  SYN_LAUNCH_CHECK("head_delta_chunks");
  // (a sequence's workgroups follow one another, a head's on one XCD where H is a multiple of 8: they read the same fragments)
  const int groups = (E + 15) / 16;
  const bool wide = (long)H * n_seqs * ((groups + 1) / 2) >= 2L * syn_compute_units();
  const dim3 grid(H, wide ? (groups + 1) / 2 : groups, n_seqs);
#define SYN_HD2(T, W, CG)                                                                                                    \
  head_delta_carry_kernel<T, W, CG><<<grid, (W + 1) * SYN_WAVE, 0, stream>>>(qkv, keys, heads, state, state_rows, seq_start, \
                                                                            seq_slot, o, H, K, D, E)
#define SYN_HD(T, W)                      \
  case T * W:                             \
    if (wide) SYN_HD2(T, W, 2);           \
    else SYN_HD2(T, W, 1);                \
    break
  switch (NT) {
    SYN_HD(1, 1); SYN_HD(1, 2); SYN_HD(1, 4); SYN_HD(2, 4); SYN_HD(3, 4); SYN_HD(4, 4);
    default: SYN_CHECK(false, "head_delta_scan: keys of %d values", D);
  }
#undef SYN_HD2
#undef SYN_HD
  SYN_LAUNCH_CHECK("head_delta_carry");
  return 0;
}

// ---------------------------------------------------------------- gated linear attention
//   z = A2 mid + bias (heads x D),  g = sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau);   S <- diag(g) S + k v^T,  o = S^T q
// q, k, v and mid (the narrow middle W_a1 h in front of the decays' second product) are columns of one projection's rows.
struct GlaArgs {
  const float* q;
  const float* k;
  const float* v;
  const float* mid;
  int ld;                    // from one token's row to the next
  const float* a2;           // [rank][H * D]: A2 transposed
  const float* a_bias;       // [H * D]
  int rank;
  float q_scale, inv_tau;
  float* state;              // [state_rows][H][D][E]
  int state_rows;
  const int* seq_start;
  const int* seq_slot;
  int H, D, E;
};

// log2 of a decay: -softplus(-z) / (tau ln 2), on the hardware's base-2 exponential and logarithm.  With w = 1 + u rounded,
// log(1 + u) = log w + (u - (w - 1)) / w up to second order in the rounding error, so that decays next to one keep their
// digits.
__device__ __forceinline__ float gla_log2_decay(float z, float inv_tau) {
  constexpr float LOG2E = 1.4426950408889634f;
  const float y = -z * LOG2E;                                   // softplus(-z) / ln 2 = log2(1 + 2^y)
  const float u = __builtin_amdgcn_exp2f(y), w = 1.f + u;
  const float sp = fmaf((u - (w - 1.f)) * LOG2E, __builtin_amdgcn_rcpf(w), __builtin_amdgcn_logf(w));
  return -(y > 30.f ? y : sp) * inv_tau;
}

#define GLA_STEP_THREADS 512
#define GLA_STEP_AHEAD 8     // rows of the state that a thread has under way

// Single tokens: a workgroup for a (head, sequence).  The state is all that moves, once in and once out, so a wave reads it
// in whole rows of VEC consecutive values a lane, and the first rows are asked for before the decays are made.  Thread =
// row group * CL + column group; the row groups' sums meet in LDS, where the head's read-out is normed and gated.
template <int VEC, typename T>
__global__ void __launch_bounds__(GLA_STEP_THREADS)
gla_step_kernel(GlaArgs a, const float* __restrict__ gain, float eps, const float* __restrict__ gate, T* __restrict__ out,
                int out_ld) {
  typedef float vec __attribute__((ext_vector_type(VEC == 1 ? 2 : VEC)));      // (one value: the first of two)
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[16];
  const int D = a.D, E = a.E, tid = threadIdx.x, head = blockIdx.x, b = blockIdx.y;
  float* qs = lds;                  // [D]
  float* ks = qs + D;               // [D]
  float* gs = ks + D;               // [D]
  float* part = gs + D;             // [row groups][E]; before that [rank shares][D]
  const int CL = E / VEC, RG = GLA_STEP_THREADS / CL;      // (the host: E a multiple of VEC, CL at most the threads)
  const int cl = tid % CL, rg = tid / CL;
  const bool on = rg < RG;
  const size_t tok = a.seq_start[b];
  int slot = a.seq_slot[b];
  if (slot < 0 || slot >= a.state_rows) slot = a.state_rows - 1;
  float* S = a.state + ((size_t)slot * a.H + head) * D * E + cl * VEC;
  auto load = [&](vec& x, int row) {
    if (on && row < D) {
      if constexpr (VEC == 1) x[0] = S[(size_t)row * E];
      else x = *(const vec*)(S + (size_t)row * E);
    }
  };
  vec s[GLA_STEP_AHEAD];
#pragma unroll
  for (int i = 0; i < GLA_STEP_AHEAD; ++i) load(s[i], rg + RG * i);
  vec v;
  if constexpr (VEC == 1) v[0] = on ? a.v[tok * a.ld + head * E + cl] : 0.f;
  else
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = on ? a.v[tok * a.ld + head * E + cl * VEC + e] : 0.f;
  // the decays: the middle's values are shared out over as many threads a channel as there are
  const int shares = GLA_STEP_THREADS / D, share = tid / D, d = tid % D, hd = head * D + d;      // (the host: D at most 256)
  if (share < shares) {
    float z = 0.f;
    for (int r0 = share; r0 < a.rank; r0 += 4 * shares) {
      float w[4], m[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = min(r0 + i * shares, a.rank - 1);
        w[i] = a.a2[(size_t)r * a.H * D + hd], m[i] = a.mid[tok * a.ld + r];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) z = fmaf(r0 + i * shares < a.rank ? w[i] : 0.f, m[i], z);
    }
    part[share * D + d] = z;
  }
  float bias = 0.f;
  if (tid < D) {
    qs[d] = a.q[tok * a.ld + hd] * a.q_scale;
    ks[d] = a.k[tok * a.ld + hd];
    bias = a.a_bias[hd];
  }
  __syncthreads();
  if (tid < D) {
    float z = bias;
    for (int i = 0; i < shares; ++i) z += part[i * D + d];
    gs[d] = __builtin_amdgcn_exp2f(gla_log2_decay(z, a.inv_tau));
  }
  __syncthreads();
  vec acc = {};
  for (int row0 = rg; row0 < D; row0 += RG * GLA_STEP_AHEAD) {
#pragma unroll
    for (int i = 0; i < GLA_STEP_AHEAD; ++i) {
      const int row = row0 + RG * i;
      if (on && row < D) {
        const float g = gs[row], kr = ks[row], qr = qs[row];
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
          s[i][e] = fmaf(g, s[i][e], kr * v[e]);
          acc[e] = fmaf(s[i][e], qr, acc[e]);
        }
        if constexpr (VEC == 1) S[(size_t)row * E] = s[i][0];
        else *(vec*)(S + (size_t)row * E) = s[i];
      }
    }
#pragma unroll
    for (int i = 0; i < GLA_STEP_AHEAD; ++i) load(s[i], row0 + RG * (GLA_STEP_AHEAD + i));
  }
  if (on) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) part[rg * E + cl * VEC + e] = acc[e];
  }
  __syncthreads();
  float o = 0.f;
  if (tid < E)
    for (int r = 0; r < RG; ++r) o += part[r * E + tid];
  const float inv = 1.f / sqrtf(block_sum(o * o, red) / (float)E + eps);
  if (tid < E) {
    const float g = gate[tok * a.ld + head * E + tid];
    out[tok * out_ld + head * E + tid] = from_f32<T>(o * inv * gain[head * E + tid] * rc_silu(g));
  }
}

// Prompts in chunks of C = 16 tokens (HDC).  With L_t = the sum of the (base 2) logarithms of the decays of the chunk's tokens up to
// t (a vector over the key channels):
//   o_t = S^T (q_t 2^L_t) + sum_(j<=t) A_tj v_j,   A_tj = sum_d q_td k_jd 2^(L_td - L_jd)
//   S'  = diag(2^L_C) S + sum_j (k_j 2^(L_C - L_j)) v_j^T
// gla_chunks_kernel makes Q 2^L, (K 2^(L_C - L))^T, A and 2^L_C for all chunks side by side; gla_carry_kernel walks a
// head's chunks with products alone, in the layout of head_delta_carry_kernel.  None of the exponents above is positive.
// A on the matrix cores is (Q 2^L) (K 2^-L)^T, whose second factor grows as the chunk's decays fall: it is taken where
// no channel loses more than 2^-GLA_SPREAD within the chunk, and else A is summed term by term.
#define GLA_SPREAD 80.f
#define GLA_RANK_PIECE 64
__host__ __device__ __forceinline__ size_t gla_chunk_floats(int NT) { return (size_t)2 * NT * 256 + 256 + 16 * NT; }

__global__ void __launch_bounds__(256)
gla_chunks_kernel(GlaArgs a, int n_seqs, float* __restrict__ work, int NT) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int LDD = 16 * NT + 1, DP = 16 * NT;
  float* qs = lds;                          // [C][LDD] queries times q_scale, zeros beyond the keys and the chunk's tokens
  float* ks = qs + HDC * LDD;               // [C][LDD]
  float* Ls = ks + HDC * LDD;               // [C][LDD] L_t
  float* mids = Ls + HDC * LDD;             // [C][GLA_RANK_PIECE]
  float* part = mids + HDC * GLA_RANK_PIECE;      // [4 waves][C][C + 1]
  float* red = part + 4 * HDC * (HDC + 1);        // [4]
  int first, n;
  if (!hd_chunk_of(blockIdx.x, a.seq_start, n_seqs, first, n)) return;      // (the whole workgroup)
  const int head = blockIdx.y, tid = threadIdx.x, wave = tid / SYN_WAVE, lane = tid % SYN_WAVE, D = a.D;
  for (int d = lane; d < DP; d += SYN_WAVE) {
    float q[HDC / 4], k[HDC / 4];
#pragma unroll
    for (int i = 0; i < HDC / 4; ++i) {
      const int t = wave + 4 * i;
      const bool in = t < n && d < D;
      const size_t at = (size_t)(first + t) * a.ld + head * D + d;
      q[i] = in ? a.q[at] * a.q_scale : 0.f, k[i] = in ? a.k[at] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < HDC / 4; ++i) qs[(wave + 4 * i) * LDD + d] = q[i], ks[(wave + 4 * i) * LDD + d] = k[i];
  }
  // the decays: a thread makes one channel's for eight tokens, then the second eight add what the first eight came to
  for (int e0 = 0; e0 < 2 * DP; e0 += 256) {
    const int e = e0 + tid, d = e % DP, t0 = e / DP * 8;
    const bool mine = e < 2 * DP, in = mine && d < D;
    float z[8];
    const float bias = in ? a.a_bias[head * D + d] : 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) z[i] = bias;
    for (int r0 = 0; r0 < a.rank; r0 += GLA_RANK_PIECE) {
      const int nr = min(GLA_RANK_PIECE, a.rank - r0);
      __syncthreads();
      for (int m = tid; m < HDC * nr; m += 256)
        mids[(m / nr) * GLA_RANK_PIECE + m % nr] = a.mid[(size_t)(first + min(m / nr, n - 1)) * a.ld + r0 + m % nr];
      __syncthreads();
      if (in)
        for (int r = 0; r < nr; r += 8) {
          float w[8];
#pragma unroll
          for (int x = 0; x < 8; ++x)
            w[x] = r + x < nr ? a.a2[(size_t)(r0 + r + x) * a.H * D + head * D + d] : 0.f;
#pragma unroll
          for (int x = 0; x < 8; ++x) {
            if (r + x < nr) {
#pragma unroll
              for (int i = 0; i < 8; ++i) z[i] = fmaf(w[x], mids[(t0 + i) * GLA_RANK_PIECE + r + x], z[i]);
            }
          }
        }
    }
    float run = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      run += (in && t0 + i < n) ? gla_log2_decay(z[i], a.inv_tau) : 0.f;      // (tokens beyond the chunk's: nothing decays)
      z[i] = run;
    }
    if (mine && t0 == 0) {
#pragma unroll
      for (int i = 0; i < 8; ++i) Ls[i * LDD + d] = z[i];
    }
    __syncthreads();      // (a channel's second eight come in the turn of its first eight or in a later one)
    if (mine && t0 != 0) {
      const float before = Ls[7 * LDD + d];
#pragma unroll
      for (int i = 0; i < 8; ++i) Ls[(8 + i) * LDD + d] = before + z[i];
    }
  }
  __syncthreads();
  float spread = 0.f;
  for (int d = tid; d < DP; d += 256) spread = fmaxf(spread, -Ls[(HDC - 1) * LDD + d]);
  spread = wave_max(spread);
  if (lane == 0) red[wave] = spread;
  __syncthreads();
  spread = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  const bool on_cores = spread <= GLA_SPREAD;                                  // (the same for the whole workgroup)
  float* wf = work + ((size_t)blockIdx.x * a.H + head) * gla_chunk_floats(NT);
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  // fragments: tile of 16 channels, lane = 16 g + m; a wave's turns are tiles wave, wave + 4, ...
  for (int e = tid; e < NT * 64; e += 256) {
    const int tile = e / 64, m = e % 16, g = (e % 64) / 16;
    hd_frag fq, ft;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = 16 * tile + 4 * g + j, dt = 16 * tile + m, t = 4 * g + j;
      fq[j] = qs[m * LDD + d] * __builtin_amdgcn_exp2f(Ls[m * LDD + d]);
      ft[j] = ks[t * LDD + dt] * __builtin_amdgcn_exp2f(Ls[(HDC - 1) * LDD + dt] - Ls[t * LDD + dt]);
    }
    ((hd_frag*)wf)[e] = fq, ((hd_frag*)wf)[NT * 64 + e] = ft;
    if (on_cores) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 16 * tile + 4 * g + j;
        acc = hd_mfma(fq[j], ks[m * LDD + d] * __builtin_amdgcn_exp2f(-Ls[m * LDD + d]), acc);
      }
    }
  }
  for (int d = tid; d < DP; d += 256) wf[2 * NT * 256 + 256 + d] = __builtin_amdgcn_exp2f(Ls[(HDC - 1) * LDD + d]);
  const int t = tid / HDC, j = tid % HDC;
  float A = 0.f;
  if (on_cores) {
#pragma unroll
    for (int i = 0; i < 4; ++i) part[(wave * HDC + 4 * (lane / 16) + i) * (HDC + 1) + lane % 16] = acc[i];
    __syncthreads();
#pragma unroll
    for (int w = 0; w < 4; ++w) A += part[(w * HDC + t) * (HDC + 1) + j];
  } else if (t >= j) {
    for (int d = 0; d < D; ++d)
      A = fmaf(qs[t * LDD + d] * ks[j * LDD + d], __builtin_amdgcn_exp2f(Ls[t * LDD + d] - Ls[j * LDD + d]), A);
  }
  wf[2 * NT * 256 + ((j / 4) * 16 + t) * 4 + j % 4] = t >= j ? A : 0.f;      // row t, k = j
}

// One chunk's operands of a wave that holds rows of the state, and of the wave that makes the outputs.
template <int TPW, int CG>
struct GlaRows {
  hd_frag q[TPW], kt[TPW];
  f32x4 gc[TPW], v[CG];      // 2^L_C of the rows 4 g + j, the values of the tokens 4 g + j in this lane's columns
};
template <int CG>
struct GlaOutput {
  hd_frag A;
  f32x4 v[CG];
};

// W waves hold TPW tiles of 16 rows of a head's state each, CG groups of 16 columns a workgroup; one more wave makes and
// stores the outputs from what the waves' rows give to Q S (through LDS, two buffers in turns: one barrier a chunk).  The
// operands are asked for STAGES chunks ahead.
template <int TPW, int W, int CG, int STAGES>
__global__ void __launch_bounds__((W + 1) * SYN_WAVE)
gla_carry_kernel(GlaArgs a, const float* __restrict__ work, float* __restrict__ o) {
  constexpr int NT = TPW * W;
  static_assert(STAGES == 2 || STAGES == 4, "the two buffers of partial sums follow the chunk's parity");
  __shared__ __attribute__((aligned(16))) f32x4 part[2][W][CG][SYN_WAVE];
  const int head = blockIdx.x, b = blockIdx.z, wave = threadIdx.x / SYN_WAVE, lane = threadIdx.x % SYN_WAVE;
  const int H = a.H, D = a.D, E = a.E, g = lane / 16, col = blockIdx.y * 16 * CG + lane % 16;
  const int s0 = a.seq_start[b], n_new = a.seq_start[b + 1] - s0;
  if (n_new <= 0) return;                            // (the whole workgroup)
  int slot = a.seq_slot[b];
  if (slot < 0 || slot >= a.state_rows) slot = a.state_rows - 1;
  const int chunk0 = s0 / HDC + b, n_chunks = (n_new + HDC - 1) / HDC;
  const float* vp = a.v + (size_t)s0 * a.ld + head * E;
  auto chunk_of = [&](int c) { return work + ((size_t)(chunk0 + c) * H + head) * gla_chunk_floats(NT); };
  auto values = [&](f32x4 (&v)[CG], int c) {
#pragma unroll
    for (int y = 0; y < CG; ++y)
#pragma unroll
      for (int j = 0; j < 4; ++j)      // (tokens beyond the last meet zeros; columns beyond are not stored)
        v[y][j] = vp[(size_t)min(c * HDC + 4 * g + j, n_new - 1) * a.ld + min(col + 16 * y, E - 1)];
  };
  // every wave walks all chunks, with one barrier a chunk
  auto walk = [&](auto& x0, auto& x1, auto& x2, auto& x3, auto&& ask, auto&& step) {
    ask(x0, 0), ask(x1, 1);
    if constexpr (STAGES == 4) ask(x2, 2), ask(x3, 3);
    for (int c = 0; c < n_chunks; c += STAGES) {
      step(x0, c, 0);
      ask(x0, c + STAGES);
      if (c + 1 < n_chunks) {
        step(x1, c + 1, 1);
        ask(x1, c + 1 + STAGES);
      }
      if constexpr (STAGES == 4) {
        if (c + 2 < n_chunks) {
          step(x2, c + 2, 0);
          ask(x2, c + 2 + STAGES);
        }
        if (c + 3 < n_chunks) {
          step(x3, c + 3, 1);
          ask(x3, c + 3 + STAGES);
        }
      }
    }
  };
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  if (wave == W) {
    float* op = o + (size_t)s0 * H * E + head * E + col;
    GlaOutput<CG> x0, x1, x2, x3;
    walk(x0, x1, x2, x3,
         [&](GlaOutput<CG>& x, int c) {
           c = min(c, n_chunks - 1);
           x.A = ((const hd_frag*)(chunk_of(c) + 2 * NT * 256))[lane];
           values(x.v, c);
         },
         [&](const GlaOutput<CG>& x, int c, int at) {
           f32x4 out[CG];
#pragma unroll
           for (int y = 0; y < CG; ++y) {
             out[y] = zero;
#pragma unroll
             for (int j = 0; j < 4; ++j) out[y] = hd_mfma(x.A[j], x.v[y][j], out[y]);
           }
           __syncthreads();
#pragma unroll
           for (int y = 0; y < CG; ++y) {
#pragma unroll
             for (int w = 0; w < W; ++w) out[y] += part[at][w][y][lane];
#pragma unroll
             for (int j = 0; j < 4; ++j) {
               const int t = c * HDC + 4 * g + j;
               if (t < n_new && col + 16 * y < E) op[(size_t)t * H * E + 16 * y] = out[y][j];
             }
           }
         });
    return;
  }
  float* Sg = a.state + ((size_t)slot * H + head) * D * E;
  f32x4 S[CG][TPW];
#pragma unroll
  for (int y = 0; y < CG; ++y)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 16 * (wave * TPW + i) + 4 * g + j, c = col + 16 * y;
        S[y][i][j] = (c < E && d < D) ? Sg[(size_t)d * E + c] : 0.f;
      }
  GlaRows<TPW, CG> x0, x1, x2, x3;
  walk(x0, x1, x2, x3,
       [&](GlaRows<TPW, CG>& x, int c) {
         c = min(c, n_chunks - 1);
         const float* wf = chunk_of(c);
         const hd_frag* kf = (const hd_frag*)wf + wave * TPW * 64 + lane;
#pragma unroll
         for (int i = 0; i < TPW; ++i) {
           x.q[i] = kf[i * 64], x.kt[i] = kf[(NT + i) * 64];
           x.gc[i] = ((const f32x4*)(wf + 2 * NT * 256 + 256))[(wave * TPW + i) * 4 + g];
         }
         values(x.v, c);
       },
       [&](const GlaRows<TPW, CG>& x, int c, int at) {
#pragma unroll
         for (int y = 0; y < CG; ++y) {
           f32x4 qs[2] = {zero, zero};
#pragma unroll
           for (int i = 0; i < TPW; ++i)
#pragma unroll
             for (int j = 0; j < 4; ++j) qs[j & 1] = hd_mfma(x.q[i][j], S[y][i][j], qs[j & 1]);
           part[at][wave][y][lane] = qs[0] + qs[1];
         }
         __syncthreads();
#pragma unroll
         for (int y = 0; y < CG; ++y) {
#pragma unroll
           for (int i = 0; i < TPW; ++i) S[y][i] *= x.gc[i];
#pragma unroll
           for (int j = 0; j < 4; ++j)
#pragma unroll
             for (int i = 0; i < TPW; ++i) S[y][i] = hd_mfma(x.kt[i][j], x.v[y][j], S[y][i]);
         }
       });
#pragma unroll
  for (int y = 0; y < CG; ++y)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 16 * (wave * TPW + i) + 4 * g + j, c = col + 16 * y;
        if (c < E && d < D) Sg[(size_t)d * E + c] = S[y][i][j];
      }
}

static int gla_check(const char* name, const GlaArgs& a, int n_seqs) {
  SYN_CHECK(n_seqs > 0 && a.H > 0 && a.D > 0 && a.E > 0 && a.rank > 0, "%s: empty input", name);
  SYN_CHECK(a.D <= RC_ROWS_MAX, "%s: keys of %d values (at most %d)", name, a.D, RC_ROWS_MAX);
  SYN_CHECK(a.ld >= a.H * max(a.D, a.E) && a.ld >= a.rank && a.state_rows > 0, "%s: rows of %d values", name, a.ld);
  return 0;
}

// floats of scratch memory of gated_linear_scan
SYN_EXPORT long syn_gated_linear_scratch(int n_tokens, int n_seqs, int H, int D) {
  return ((long)n_tokens / HDC + n_seqs) * H * (long)gla_chunk_floats(hd_tiles(D));
}

// any number of new tokens a sequence; o [n_tokens][H * E] float
SYN_EXPORT int syn_gated_linear_scan(const float* q, const float* k, const float* v, const float* mid, int ld, const float* a2,
                                     const float* a_bias, int rank, float q_scale, float inv_tau, float* state, int state_rows,
                                     const int* seq_start, const int* seq_slot, int n_seqs, int n_tokens, int H, int D, int E,
                                     float* o, float* scratch, hipStream_t stream) {
  const GlaArgs a = {q, k, v, mid, ld, a2, a_bias, rank, q_scale, inv_tau, state, state_rows, seq_start, seq_slot, H, D, E};
  if (int rc = gla_check("gated_linear_scan", a, n_seqs)) return rc;
  SYN_CHECK(n_tokens > 0 && scratch && (uintptr_t)scratch % 16 == 0, "gated_linear_scan: the scratch memory is not aligned");
  const int NT = hd_tiles(D), chunks = n_tokens / HDC + n_seqs;
  const size_t bytes = (3 * HDC * (16 * NT + 1) + HDC * GLA_RANK_PIECE + 4 * HDC * (HDC + 1) + 4) * sizeof(float);
  gla_chunks_kernel<<<dim3(chunks, H), 256, bytes, stream>>>(a, n_seqs, scratch, NT);
  SYN_LAUNCH_CHECK("gla_chunks");
  const int groups = (E + 15) / 16;
  const bool wide = (long)H * n_seqs * ((groups + 1) / 2) >= 2L * syn_compute_units();
  const dim3 grid(H, wide ? (groups + 1) / 2 : groups, n_seqs);
#define SYN_GLA2(T, W, CG) gla_carry_kernel<T, W, CG, (T) <= 2 ? 4 : 2><<<grid, (W + 1) * SYN_WAVE, 0, stream>>>(a, scratch, o)
#define SYN_GLA(T, W)                 \
  case T * W:                         \
    if (wide) SYN_GLA2(T, W, 2);      \
    else SYN_GLA2(T, W, 1);           \
    break
  switch (NT) {
    SYN_GLA(1, 1); SYN_GLA(1, 2); SYN_GLA(1, 4); SYN_GLA(2, 4); SYN_GLA(3, 4); SYN_GLA(4, 4);
    default: SYN_CHECK(false, "gated_linear_scan: keys of %d values", D);
  }
#undef SYN_GLA2
#undef SYN_GLA
  SYN_LAUNCH_CHECK("gla_carry");
  return 0;
}

// one new token a sequence; out [n_seqs] rows of out_ld values: each head's read-out over its root mean square, times gain
// [H * E], times silu(gate) (columns of the projection's rows)
SYN_EXPORT int syn_gated_linear_step(const float* q, const float* k, const float* v, const float* mid, int ld, const float* a2,
                                     const float* a_bias, int rank, float q_scale, float inv_tau, float* state, int state_rows,
                                     const int* seq_start, const int* seq_slot, int n_seqs, int H, int D, int E,
                                     const float* gain, float eps, const float* gate, void* out, int out_ld, int out_is_f32,
                                     hipStream_t stream) {
  const GlaArgs a = {q, k, v, mid, ld, a2, a_bias, rank, q_scale, inv_tau, state, state_rows, seq_start, seq_slot, H, D, E};
  if (int rc = gla_check("gated_linear_step", a, n_seqs)) return rc;
  SYN_CHECK(E <= GLA_STEP_THREADS, "gated_linear_step: values of %d (at most %d)", E, GLA_STEP_THREADS);
  SYN_CHECK(gain && gate && out && out_ld >= H * E, "gated_linear_step: result rows of %d values", out_ld);
  const bool four = E % 4 == 0 && (uintptr_t)state % 16 == 0;
  const int row_groups = GLA_STEP_THREADS / (four ? E / 4 : E);
  const size_t bytes = (3 * (size_t)D + (size_t)max(row_groups * E, GLA_STEP_THREADS)) * sizeof(float);
  const dim3 grid(H, n_seqs);
#define SYN_GLAS(VEC, T) gla_step_kernel<VEC, T><<<grid, GLA_STEP_THREADS, bytes, stream>>>(a, gain, eps, gate, (T*)out, out_ld)
  if (out_is_f32) {
    if (four) SYN_GLAS(4, float); else SYN_GLAS(1, float);
  } else {
    if (four) SYN_GLAS(4, bf16); else SYN_GLAS(1, bf16);
  }
#undef SYN_GLAS
  SYN_LAUNCH_CHECK("gated_linear_step");
  return 0;
}

// ---------------------------------------------------------------- two softmax maps over the same values
// a [N][G][2][Rq][E]: for each kv head the heads' results of the first map, then of the second (the order in which
// grouped-query attention over 2 G key heads leaves them); out [N][G * Rq][E] = rms_norm(a1 - lambda a2) * post.
// One wave a (token, head).
template <typename T>
__global__ void diff_heads_kernel(const T* __restrict__ a, T* __restrict__ out, float lambda, float eps, float post,
                                  int n_items, int G, int Rq, int E) {
  const int item = blockIdx.x * (blockDim.x / SYN_WAVE) + threadIdx.x / SYN_WAVE;
  if (item >= n_items) return;
  const int lane = threadIdx.x % SYN_WAVE;
  const int H = G * Rq, tok = item / H, h = item % H, g = h / Rq, r = h % Rq;
  const T* a1 = a + (((size_t)tok * G + g) * 2 * Rq + r) * E;
  const T* a2 = a1 + (size_t)Rq * E;
  float ss = 0.f;
  for (int d = lane; d < E; d += SYN_WAVE) {
    const float v = to_f32<T>(a1[d]) - lambda * to_f32<T>(a2[d]);
    ss = fmaf(v, v, ss);
  }
  const float f = post / sqrtf(wave_sum(ss) / (float)E + eps);
  for (int d = lane; d < E; d += SYN_WAVE)
    out[((size_t)tok * H + h) * E + d] = from_f32<T>((to_f32<T>(a1[d]) - lambda * to_f32<T>(a2[d])) * f);
}

SYN_EXPORT int syn_diff_heads(const void* a, void* out, int is_f32, float lambda, float eps, float post, int n_tokens, int G,
                              int Rq, int E, hipStream_t stream) {
  SYN_CHECK(n_tokens > 0 && G > 0 && Rq > 0 && E > 0, "diff_heads: empty input");
  const int wpb = 4, items = n_tokens * G * Rq, grid = (items + wpb - 1) / wpb;
  if (is_f32)
    diff_heads_kernel<float><<<grid, wpb * SYN_WAVE, 0, stream>>>((const float*)a, (float*)out, lambda, eps, post, items, G, Rq, E);
  else
    diff_heads_kernel<bf16><<<grid, wpb * SYN_WAVE, 0, stream>>>((const bf16*)a, (bf16*)out, lambda, eps, post, items, G, Rq, E);
  SYN_LAUNCH_CHECK("diff_heads");
  return 0;
}
