// Layers that carry a fixed-size state from token to token: the short causal convolution over time
// (per channel, a few taps) and the gated delta rule (per head a matrix S [key dim, value dim] that
// decays per key channel, is corrected towards the new value along the new key, and is read with the
// query).  States are float32 and live in the cache's per-slot storage; a step brings any number of
// tokens per sequence on top of what the state holds.  All arithmetic here is float32.
#include <math.h>

#include "api.h"
#include "common.h"

__device__ __forceinline__ float rb_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float rb_softplus(float v) { return v > 20.0f ? v : log1pf(expf(v)); }

// ---------------------------------------------------------------- short convolution
// y[t, c] = (residual ? x[t, c] : 0) + sum_d w[c, taps - 1 - d] * x[t - d, c], d = 0 .. taps - 1, where rows
// before the step's first come from the sequence's state (its last taps - 1 inputs, oldest first) and rows
// before the sequence's start are zero (the state of a fresh slot is zero).  act 1: silu on the result.
// Afterwards the state holds the last taps - 1 inputs again.  One launch: workgroups that walk 16 rows each of the
// tokens that need rows of the step only, and a workgroup per sequence that walks the step's first taps - 1 tokens with
// the old state in registers and then writes the new state, so that whoever reads the state is also who writes it.
#define SC_MAX_TAPS 16
#define SC_TILE 16             // rows of the step that a workgroup walks
template <typename TO>
__global__ void short_conv_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ bias,
                                  const float* __restrict__ bias_out, const float* __restrict__ w, int taps,
                                  float* __restrict__ state, const int32_t* __restrict__ tok_pos,
                                  const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ cu_seqlens,
                                  const int32_t* __restrict__ slots, TO* __restrict__ out, size_t out_stride,
                                  int residual, int act, int channels, int n_tokens, int n_tiles) {
  const int keep = taps - 1;
  if ((int)blockIdx.x < n_tiles) {
    // SC_TILE rows of the packed step, walked with the window (the last taps - 1 inputs) in registers: one new row a
    // token.  Rows that are among a sequence's first taps - 1 of the step belong to the sequence's workgroup; after such
    // a row (and at the tile's start) the window is read anew.
    const int r0 = blockIdx.x * SC_TILE;
    const int r1 = r0 + SC_TILE < n_tokens ? r0 + SC_TILE : n_tokens;
    for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < channels; c += gridDim.y * blockDim.x) {
      float win[SC_MAX_TAPS], wt[SC_MAX_TAPS];
#pragma unroll
      for (int j = 0; j < SC_MAX_TAPS; ++j) {
        win[j] = 0.f;
        wt[j] = j < keep ? w[(size_t)c * taps + j] : 0.f;
      }
      const float w_cur = w[(size_t)c * taps + keep];
      const float bc = bias ? bias[c] : 0.f, bo = bias_out ? bias_out[c] : 0.f;
      bool have = false;
      for (int t = r0; t < r1; ++t) {
        if (t - cu_seqlens[tok_seq[t]] < keep) {             // the sequence's workgroup takes it
          have = false;
          continue;
        }
        if (!have) {
#pragma unroll
          for (int j = 0; j < SC_MAX_TAPS; ++j)
            if (j < keep) win[j] = x[(size_t)(t - keep + j) * x_stride + c] + bc;
          have = true;
        }
        const float cur = x[(size_t)t * x_stride + c] + bc;
        float acc = residual ? cur : bo;
        acc = fmaf(w_cur, cur, acc);
#pragma unroll
        for (int j = 0; j < SC_MAX_TAPS; ++j) acc = fmaf(wt[j], win[j], acc);
#pragma unroll
        for (int j = 0; j < SC_MAX_TAPS - 1; ++j) win[j] = j + 1 < keep ? win[j + 1] : win[j];
#pragma unroll
        for (int j = 0; j < SC_MAX_TAPS; ++j)
          if (j == keep - 1) win[j] = cur;
        if (act == 1) acc = acc * rb_sigmoid(acc);
        Num<TO>::store(out + (size_t)t * out_stride + c, acc);
      }
    }
    return;
  }
  const int b = blockIdx.x - n_tiles;
  const int row0 = cu_seqlens[b], n = cu_seqlens[b + 1] - row0;
  float* st = state + (size_t)slots[b] * keep * channels;
  const int first = n < keep ? n : keep;
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < channels; c += gridDim.y * blockDim.x) {
    float win[SC_MAX_TAPS], wt[SC_MAX_TAPS];                 // the last `keep` inputs, oldest first; their weights
#pragma unroll
    for (int j = 0; j < SC_MAX_TAPS; ++j) {
      win[j] = j < keep ? st[(size_t)j * channels + c] : 0.f;
      wt[j] = j < keep ? w[(size_t)c * taps + j] : 0.f;
    }
    const float w_cur = w[(size_t)c * taps + keep];
    const float bc = bias ? bias[c] : 0.f, bo = bias_out ? bias_out[c] : 0.f;
    float nxt = first > 0 ? x[(size_t)row0 * x_stride + c] + bc : 0.f;
    __builtin_amdgcn_sched_barrier(0);                       // state, weights and the first row: one trip to memory together
    for (int i = 0; i < first; ++i) {
      const float cur = nxt;
      if (i + 1 < first) nxt = x[(size_t)(row0 + i + 1) * x_stride + c] + bc;
      float acc = residual ? cur : bo;
      acc = fmaf(w_cur, cur, acc);
#pragma unroll
      for (int j = 0; j < SC_MAX_TAPS; ++j) acc = fmaf(wt[j], win[j], acc);
#pragma unroll
      for (int j = 0; j < SC_MAX_TAPS - 1; ++j) win[j] = j + 1 < keep ? win[j + 1] : win[j];
#pragma unroll
      for (int j = 0; j < SC_MAX_TAPS; ++j)
        if (j == keep - 1) win[j] = cur;
      if (act == 1) acc = acc * rb_sigmoid(acc);
      Num<TO>::store(out + (size_t)(row0 + i) * out_stride + c, acc);
    }
#pragma unroll
    for (int j = 0; j < SC_MAX_TAPS; ++j)
      if (j < keep) st[(size_t)j * channels + c] = n > keep ? x[(size_t)(row0 + n - keep + j) * x_stride + c] + bc : win[j];
  }
}

// The same for four channels a thread (16-byte loads) and few taps (KEEP = taps - 1 of them before the current one), so that no
// predicate stands at a tap.
template <int KEEP>
__device__ __forceinline__ void conv4(float (&win)[KEEP][4], const float (&wt)[KEEP][4], const float (&w_cur)[4], const float4& now,
                                      const float (&bo)[4], int residual, int act, float (&acc)[4]) {
  const float cur[4] = {now.x, now.y, now.z, now.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    float a = fmaf(w_cur[i], cur[i], residual ? cur[i] : bo[i]);
#pragma unroll
    for (int j = 0; j < KEEP; ++j) a = fmaf(wt[j][i], win[j][i], a);
#pragma unroll
    for (int j = 0; j + 1 < KEEP; ++j) win[j][i] = win[j + 1][i];
    win[KEEP - 1][i] = cur[i];
    acc[i] = act == 1 ? a * rb_sigmoid(a) : a;
  }
}
__device__ __forceinline__ void conv_store4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void conv_store4(bf16_t* p, const float (&v)[4]) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
}
template <typename TO, int KEEP>
__global__ __launch_bounds__(256) void short_conv_vec_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ bias,
                                                             const float* __restrict__ bias_out, const float* __restrict__ w,
                                                             float* __restrict__ state, const int32_t* __restrict__ tok_seq,
                                                             const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots,
                                                             TO* __restrict__ out, size_t out_stride, int residual, int act, int channels,
                                                             int n_tokens, int n_tiles) {
  const int c = 4 * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= channels) return;
  float wt[KEEP][4], w_cur[4], bc[4], bo[4], win[KEEP][4], acc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
#pragma unroll
    for (int j = 0; j < KEEP; ++j) wt[j][i] = w[(size_t)(c + i) * (KEEP + 1) + j];
    w_cur[i] = w[(size_t)(c + i) * (KEEP + 1) + KEEP];
    bc[i] = bias ? bias[c + i] : 0.f;
    bo[i] = bias_out ? bias_out[c + i] : 0.f;
  }
  auto row = [&](size_t t) {
    float4 v = *reinterpret_cast<const float4*>(x + t * x_stride + c);
    return make_float4(v.x + bc[0], v.y + bc[1], v.z + bc[2], v.w + bc[3]);
  };
  auto put = [&](int j, const float4& v) {
    win[j][0] = v.x, win[j][1] = v.y, win[j][2] = v.z, win[j][3] = v.w;
  };
  if ((int)blockIdx.x < n_tiles) {
    const int r0 = blockIdx.x * SC_TILE, r1 = r0 + SC_TILE < n_tokens ? r0 + SC_TILE : n_tokens;
    if (tok_seq[r0] == tok_seq[r1 - 1] && r1 - r0 == SC_TILE && r0 - cu_seqlens[tok_seq[r0]] >= KEEP) {
      // a whole tile inside one sequence's piece: all its rows are asked for together
      float4 rows[SC_TILE];
#pragma unroll
      for (int j = 0; j < KEEP; ++j) put(j, row((size_t)(r0 - KEEP + j)));
#pragma unroll
      for (int t = 0; t < SC_TILE; ++t) rows[t] = row((size_t)(r0 + t));
#pragma unroll
      for (int t = 0; t < SC_TILE; ++t) {
        conv4<KEEP>(win, wt, w_cur, rows[t], bo, residual, act, acc);
        conv_store4(out + (size_t)(r0 + t) * out_stride + c, acc);
      }
      return;
    }
    bool have = false;
    for (int t = r0; t < r1; ++t) {
      if (t - cu_seqlens[tok_seq[t]] < KEEP) {               // the sequence's workgroup takes it
        have = false;
        continue;
      }
      if (!have) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) put(j, row((size_t)(t - KEEP + j)));
        have = true;
      }
      conv4<KEEP>(win, wt, w_cur, row((size_t)t), bo, residual, act, acc);
      conv_store4(out + (size_t)t * out_stride + c, acc);
    }
    return;
  }
  const int b = blockIdx.x - n_tiles;
  const int row0 = cu_seqlens[b], n = cu_seqlens[b + 1] - row0;
  float* st = state + (size_t)slots[b] * KEEP * channels + c;
  const int first = n < KEEP ? n : KEEP;
#pragma unroll
  for (int j = 0; j < KEEP; ++j) put(j, *reinterpret_cast<const float4*>(st + (size_t)j * channels));
  float4 rows[KEEP];
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (i < first) rows[i] = row((size_t)(row0 + i));
  __builtin_amdgcn_sched_barrier(0);                         // state, weights and rows: one trip to memory together
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (i < first) {
      conv4<KEEP>(win, wt, w_cur, rows[i], bo, residual, act, acc);
      conv_store4(out + (size_t)(row0 + i) * out_stride + c, acc);
    }
  if (n <= 0) return;
#pragma unroll
  for (int j = 0; j < KEEP; ++j) {
    const float4 v = n > KEEP ? row((size_t)(row0 + n - KEEP + j)) : make_float4(win[j][0], win[j][1], win[j][2], win[j][3]);
    *reinterpret_cast<float4*>(st + (size_t)j * channels) = v;
  }
}

extern "C" int rb_short_conv(const float* x, long long x_stride, const float* w, int taps, float* state,
                             const int32_t* tok_pos, const int32_t* tok_seq, const int32_t* cu_seqlens,
                             const int32_t* slots, void* out, long long out_stride, int out_dtype, int residual,
                             int act, int n_tokens, int n_seqs, int channels, void* stream) {
  RB_RECORDED(rb_short_conv(x, x_stride, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots, out, out_stride, out_dtype,
                            residual, act, n_tokens, n_seqs, channels, stream));
  return rb_short_conv_bias(x, x_stride, nullptr, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots, out, out_stride, out_dtype,
                            residual, act, n_tokens, n_seqs, channels, stream);
}

// The same on x + bias (bias float32 [C], null: none): the bias belongs to the inputs, so the state holds them with it and
// rows before a sequence's start stay zero.
extern "C" int rb_short_conv_bias(const float* x, long long x_stride, const float* bias, const float* w, int taps, float* state,
                                  const int32_t* tok_pos, const int32_t* tok_seq, const int32_t* cu_seqlens,
                                  const int32_t* slots, void* out, long long out_stride, int out_dtype, int residual,
                                  int act, int n_tokens, int n_seqs, int channels, void* stream) {
  RB_RECORDED(rb_short_conv_bias(x, x_stride, bias, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots, out, out_stride, out_dtype,
                                 residual, act, n_tokens, n_seqs, channels, stream));
  return rb_short_conv_biases(x, x_stride, bias, nullptr, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots, out, out_stride, out_dtype,
                              residual, act, n_tokens, n_seqs, channels, stream);
}

// The same with a bias on the convolution's result as well (bias_out float32 [C], null: none; not with residual), in front of the
// activation; the state knows nothing of it.
extern "C" int rb_short_conv_biases(const float* x, long long x_stride, const float* bias, const float* bias_out, const float* w, int taps,
                                    float* state, const int32_t* tok_pos, const int32_t* tok_seq, const int32_t* cu_seqlens,
                                    const int32_t* slots, void* out, long long out_stride, int out_dtype, int residual, int act,
                                    int n_tokens, int n_seqs, int channels, void* stream) {
  RB_RECORDED(rb_short_conv_biases(x, x_stride, bias, bias_out, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots, out, out_stride,
                                   out_dtype, residual, act, n_tokens, n_seqs, channels, stream));
  RB_REQUIRE(bias_out == nullptr || !residual, "rb_short_conv: a bias on the result goes without the residual");
  RB_REQUIRE(n_tokens >= 0 && n_seqs >= 0 && channels > 0 && taps >= 1 && taps - 1 <= SC_MAX_TAPS,
             "rb_short_conv: bad sizes T=%d B=%d C=%d taps=%d (at most %d)", n_tokens, n_seqs, channels, taps, SC_MAX_TAPS + 1);
  RB_REQUIRE(x_stride >= channels && out_stride >= channels, "rb_short_conv: a row stride is shorter than the channels");
  RB_REQUIRE(taps == 1 || state != nullptr, "rb_short_conv: %d taps need a state", taps);
  RB_REQUIRE(act == 0 || act == 1, "rb_short_conv: unknown activation %d", act);
  if (n_tokens == 0) return 0;
  const int n_tiles = (n_tokens + SC_TILE - 1) / SC_TILE;
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (taps >= 2 && taps <= 4 && channels % 4 == 0 && x_stride % 4 == 0 && out_stride % 4 == 0 && aligned(x) && aligned(state) && aligned(out) &&
      (out_dtype == RB_F32 || out_dtype == RB_BF16)) {
    const int threads = n_tokens <= n_seqs ? RB_WAVE : 256;   // single tokens: few workgroups, so small ones
    const dim3 vgrid((n_tokens <= n_seqs ? 0 : n_tiles) + n_seqs, (channels / 4 + threads - 1) / threads);
    const int vtiles = n_tokens <= n_seqs ? 0 : n_tiles;
    RB_REQUIRE(vgrid.y <= 65535, "rb_short_conv: %d channels are too many", channels);
#define SC_GO(TO, KEEP)                                                                                                            \
  short_conv_vec_kernel<TO, KEEP><<<vgrid, threads, 0, (hipStream_t)stream>>>(x, (size_t)x_stride, bias, bias_out, w, state, tok_seq,  \
                                                                              cu_seqlens, slots, (TO*)out, (size_t)out_stride, residual, \
                                                                              act, channels, n_tokens, vtiles)
#define SC_BY_TAPS(TO)                \
  do {                                \
    if (taps == 2) SC_GO(TO, 1);      \
    else if (taps == 3) SC_GO(TO, 2); \
    else SC_GO(TO, 3);                \
  } while (0)
    if (out_dtype == RB_F32) SC_BY_TAPS(float);
    else SC_BY_TAPS(bf16_t);
#undef SC_BY_TAPS
#undef SC_GO
    RB_LAUNCH_CHECK();
    return 0;
  }
  dim3 grid(n_tiles + (taps > 1 ? n_seqs : 0), (channels + 255) / 256 < 64 ? (channels + 255) / 256 : 64);
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == RB_F32)
    short_conv_kernel<float><<<grid, 256, 0, s>>>(x, (size_t)x_stride, bias, bias_out, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots,
                                                  (float*)out, (size_t)out_stride, residual, act, channels, n_tokens, n_tiles);
  else if (out_dtype == RB_BF16)
    short_conv_kernel<bf16_t><<<grid, 256, 0, s>>>(x, (size_t)x_stride, bias, bias_out, w, taps, state, tok_pos, tok_seq, cu_seqlens, slots,
                                                   (bf16_t*)out, (size_t)out_stride, residual, act, channels, n_tokens, n_tiles);
  else
    RB_REQUIRE(false, "rb_short_conv: unknown dtype %d", out_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- what enters a recurrence
// Per token, in place.  The q and k heads (n_kv of each, `dim` numbers): unit 1 makes each a unit vector,
// x / sqrt(sum x^2 + unit_eps); q is also multiplied by q_scale (unit 0: only that).  The a_cols numbers of a row of
// `a` become decays, a_cols being H (one per head) or H * dim (one per head and key channel), h = i / (a_cols / H):
//   decay 0:  exp(-exp(a_log[h]) * softplus(a + bias[i]))
//   decay 1:  sigmoid(a + bias[i]) ^ (1 / tau), computed as exp(-softplus(-(a + bias[i])) / tau)
//   decay 2:  exp(-exp(a + bias[i]))
// beta[t, h] = sigmoid(b[t, h]) where b_in is given.
__global__ __launch_bounds__(1024) void recurrence_prep_kernel(float* __restrict__ qk, size_t qk_stride, int n_kv, int dim, int unit,
                                  float* __restrict__ a, size_t a_stride, int a_cols, int decay, const float* __restrict__ bias,
                                  const float* __restrict__ a_log, float tau, int n_heads,
                                  const float* __restrict__ b_in, size_t b_stride, float* __restrict__ beta,
                                  float q_scale, float unit_eps) {
  const int t = blockIdx.x;
  const int lane = threadIdx.x & (RB_WAVE - 1);
  const int wave = threadIdx.x / RB_WAVE, n_waves = blockDim.x / RB_WAVE;
  float* row = qk + (size_t)t * qk_stride;
  if (unit) {
    for (int v = wave; v < 2 * n_kv; v += n_waves) {           // the q heads, then the k heads
      float* p = row + (size_t)v * dim;
      float ss = 0.f;
      for (int i = lane; i < dim; i += RB_WAVE) ss = fmaf(p[i], p[i], ss);
      ss = wave_sum(ss);
      const float f = (v < n_kv ? q_scale : 1.0f) / sqrtf(ss + unit_eps);
      for (int i = lane; i < dim; i += RB_WAVE) p[i] *= f;
    }
  } else if (q_scale != 1.0f) {
    for (int i = threadIdx.x; i < n_kv * dim; i += blockDim.x) row[i] *= q_scale;
  }
  float* ar = a + (size_t)t * a_stride;
  const int per_head = a_cols / n_heads;
  for (int i = threadIdx.x; i < a_cols; i += blockDim.x) {
    const float z = ar[i] + (bias ? bias[i] : 0.f);
    if (decay == 0)
      ar[i] = expf(-expf(a_log[i / per_head]) * rb_softplus(z));
    else if (decay == 1)
      ar[i] = expf(-rb_softplus(-z) / tau);
    else
      ar[i] = expf(-expf(z));
  }
  if (b_in)
    for (int h = threadIdx.x; h < n_heads; h += blockDim.x) beta[(size_t)t * n_heads + h] = rb_sigmoid(b_in[(size_t)t * b_stride + h]);
}

extern "C" int rb_recurrence_prep(float* qk, long long qk_stride, int n_kv_heads, int dim, int unit, float q_scale, float unit_eps,
                                  float* a, long long a_stride, int a_cols, int decay, const float* bias, const float* a_log,
                                  float tau, int n_heads, const float* b_in, long long b_stride, float* beta, int n_tokens,
                                  void* stream) {
  RB_RECORDED(rb_recurrence_prep(qk, qk_stride, n_kv_heads, dim, unit, q_scale, unit_eps, a, a_stride, a_cols, decay, bias, a_log,
                                 tau, n_heads, b_in, b_stride, beta, n_tokens, stream));
  RB_REQUIRE(n_tokens >= 0 && n_kv_heads >= 0 && n_heads > 0 && dim > 0, "rb_recurrence_prep: bad sizes");      // no q/k heads: the decays alone
  RB_REQUIRE(a_cols == n_heads || a_cols == n_heads * dim, "rb_recurrence_prep: %d decays a token for %d heads of %d", a_cols,
             n_heads, dim);
  RB_REQUIRE(qk_stride >= 2LL * n_kv_heads * dim && a_stride >= a_cols && (b_in == nullptr || b_stride >= n_heads),
             "rb_recurrence_prep: a row stride is too short");
  RB_REQUIRE((decay == 0 && a_log != nullptr) || (decay == 1 && tau > 0.f) || decay == 2,
             "rb_recurrence_prep: decay %d lacks its constants", decay);
  RB_REQUIRE(b_in == nullptr || beta != nullptr, "rb_recurrence_prep: beta has nowhere to go");
  if (n_tokens == 0) return 0;
  // a step of few tokens has few workgroups, and a token's heads are a chain of trips to memory for each wave: more waves then
  const int threads = n_tokens < 2 * rb_compute_units() ? 1024 : 256;
  recurrence_prep_kernel<<<n_tokens, threads, 0, (hipStream_t)stream>>>(qk, (size_t)qk_stride, n_kv_heads, dim, unit, a, (size_t)a_stride,
                                                                    a_cols, decay, bias, a_log, tau, n_heads, b_in, (size_t)b_stride,
                                                                    beta, q_scale, unit_eps);
  RB_LAUNCH_CHECK();
  return 0;
}

// The gated delta rule with a decay per key channel: unit vectors, decay 0 on H * dim numbers, beta.
extern "C" int rb_delta_prep(float* qk, long long qk_stride, int n_kv_heads, int dim, float* a, long long a_stride, const float* dt_bias,
                             const float* a_log, int n_heads, const float* b_in, long long b_stride, float* beta,
                             float q_scale, float unit_eps, int n_tokens, void* stream) {
  RB_RECORDED(rb_delta_prep(qk, qk_stride, n_kv_heads, dim, a, a_stride, dt_bias, a_log, n_heads, b_in, b_stride, beta, q_scale,
                            unit_eps, n_tokens, stream));
  return rb_recurrence_prep(qk, qk_stride, n_kv_heads, dim, 1, q_scale, unit_eps, a, a_stride, n_heads * dim, 0, dt_bias, a_log, 1.0f,
                            n_heads, b_in, b_stride, beta, n_tokens, stream);
}

// ---------------------------------------------------------------- gated delta rule: the recurrence
// Per sequence and head, token after token:
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// The columns of S (one per value channel) do not meet: a column is held by RG lanes, each with DKL of its rows in
// registers; the dot products over the rows are finished among the RG lanes by moves inside a row of lanes.  A workgroup is one wave
// and holds 64 / RG columns.  Tokens go by in chunks of CH: q, k, g, v and beta of a chunk lie in LDS for all lanes, and
// the next chunk's loads are in flight (in registers) while the current one is computed, so that a token costs its
// arithmetic and no trip to memory; the chunk's outputs leave through LDS as whole rows.  The state is read once and
// written once.
// The sum over each group of RG neighbouring lanes (RG = 4, 8 or 16), in every lane of the group, by moves inside a
// row of 16 lanes (no trip through LDS): the two swaps inside a quad, then the mirror of a half row, then of a row.
template <int RG>
__device__ __forceinline__ float lanes_sum(float v) {
  static_assert(RG == 4 || RG == 8 || RG == 16, "groups of 4, 8 or 16 lanes");
  v += __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));   // quad_perm [1,0,3,2]
  v += __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));   // quad_perm [2,3,0,1]
  if (RG >= 8) v += __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));   // row_half_mirror
  if (RG >= 16) v += __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));  // row_mirror
  return v;
}

// MODE 0: as above; 1: the read before the write, with a bonus (see below); 2: q, k and v go through silu as they are fetched;
// 3: a selective scan: every token has a step size dt = softplus(dt_in + dt_bias[h]) per head, from which the decay and the
// weight of the write come, and its value passes to the read-out with a weight of the head:
//   S <- exp(-exp(a_log[h]) dt) S + dt k v^T;  o = S^T q + d[h] v
struct SelectiveArgs {
  const float* dt_in;
  size_t dt_stride;
  const float *dt_bias, *a_log, *d;
};
template <int DKL, int RG, int CH, int MODE>
__global__ __launch_bounds__(RB_WAVE) void delta_rule_kernel(
    const float* __restrict__ q, const float* __restrict__ k, size_t qk_stride, const float* __restrict__ v,
    size_t v_stride, const float* __restrict__ g, size_t g_stride, const float* __restrict__ beta, float* __restrict__ state,
    const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots, float* __restrict__ out, int n_heads,
    int n_kv, int dim, int vdim, int g_per_head, const float* __restrict__ bonus, SelectiveArgs sel) {
  constexpr bool BONUS = MODE == 1, SELECTIVE = MODE == 3;
  constexpr int COLS = RB_WAVE / RG;
  constexpr int DK = DKL * RG;               // rows held, >= dim; rows beyond dim stay zero
  constexpr int NQ = DK * CH / RB_WAVE;      // q (or k, or g) values of a chunk per lane
  constexpr int NV = (COLS * CH + RB_WAVE - 1) / RB_WAVE;
  __shared__ float sq[CH][DK], sk[CH][DK], sg[SELECTIVE ? 1 : CH][SELECTIVE ? CH : DK], sv[CH][COLS], so[CH][COLS], sb[CH];
  const int b = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x;
  const int col0 = blockIdx.z * COLS;
  const int col = col0 + lane / RG;
  const int rg = lane % RG;
  const bool on = col < vdim;
  const int kvh = h / (n_heads / n_kv);
  const int row0 = cu_seqlens[b], n = cu_seqlens[b + 1] - row0;
  // the state is kept column by column, [slots, H, vdim, dim]: a lane's rows are DKL numbers in a row and a wave's
  // columns one piece of memory (with S as rows a wave of four columns used a quarter of every line it touched)
  float* S = state + (((size_t)slots[b] * n_heads + h) * vdim + (on ? col : 0)) * dim;
  float s[DKL];
  const bool quads = dim % 4 == 0 && DKL % 4 == 0 && (reinterpret_cast<uintptr_t>(state) & 15) == 0;
  if (quads) {
#pragma unroll
    for (int i = 0; i < DKL; i += 4) {
      const int r = rg * DKL + i;
      const float4 v4 = (on && r < dim) ? *reinterpret_cast<const float4*>(S + r) : make_float4(0.f, 0.f, 0.f, 0.f);
      s[i] = v4.x;
      s[i + 1] = v4.y;
      s[i + 2] = v4.z;
      s[i + 3] = v4.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < DKL; ++i) {
      const int r = rg * DKL + i;
      s[i] = (on && r < dim) ? S[r] : 0.f;
    }
  }
  // BONUS: the read-out sees the state as it was before the token, and the token's own k v^T times a weight per key
  // channel: o = S^T q + v sum_i bonus_i k_i q_i;  then S <- diag(g) S + k v^T
  float ub[DKL];
#pragma unroll
  for (int i = 0; i < DKL; ++i) {
    const int r = rg * DKL + i;
    ub[i] = (BONUS && r < dim) ? bonus[(size_t)h * dim + r] : 0.f;
  }
  float rq[NQ], rk[NQ], rgt[SELECTIVE ? 1 : NQ], rv[NV], rb = 0.f;
  const float rate = SELECTIVE ? expf(sel.a_log[h]) : 0.f, dt_bias = SELECTIVE ? sel.dt_bias[h] : 0.f, pass = SELECTIVE ? sel.d[h] : 0.f;
  auto fetch = [&](int t0) {
    const int nt = n - t0 < CH ? n - t0 : CH;
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      const int e = lane + RB_WAVE * j, tt = e / DK, i = e - tt * DK;
      const bool in = tt < nt && i < dim;
      const size_t t = (size_t)(row0 + t0 + tt);
      rq[j] = in ? q[t * qk_stride + (size_t)kvh * dim + i] : 0.f;
      rk[j] = in ? k[t * qk_stride + (size_t)kvh * dim + i] : 0.f;
      if (!SELECTIVE) rgt[j] = in ? (g_per_head ? g[t * g_stride + h] : g[t * g_stride + (size_t)h * dim + i]) : 0.f;
      if (MODE == 2) {
        rq[j] *= rb_sigmoid(rq[j]);
        rk[j] *= rb_sigmoid(rk[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int e = lane + RB_WAVE * j, tt = e / COLS, c = e - tt * COLS;
      rv[j] = (tt < nt && col0 + c < vdim) ? v[(size_t)(row0 + t0 + tt) * v_stride + (size_t)h * vdim + col0 + c] : 0.f;
      if (MODE == 2) rv[j] *= rb_sigmoid(rv[j]);
    }
    if (SELECTIVE)                                     // the step's raw number: what it becomes is made when the chunk goes to LDS
      rb = lane < nt ? sel.dt_in[(size_t)(row0 + t0 + lane) * sel.dt_stride + h] : 0.f;
    else
      rb = (beta && lane < nt) ? beta[(size_t)(row0 + t0 + lane) * n_heads + h] : 0.f;
  };
  if (n > 0) fetch(0);
  for (int t0 = 0; t0 < n; t0 += CH) {
    const int nt = n - t0 < CH ? n - t0 : CH;
    __syncthreads();                                   // the chunk before has been read and its outputs are out
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      const int e = lane + RB_WAVE * j, tt = e / DK, i = e - tt * DK;
      sq[tt][i] = rq[j];
      sk[tt][i] = rk[j];
      if (!SELECTIVE) sg[tt][i] = rgt[j];
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int e = lane + RB_WAVE * j;
      if (e < COLS * CH) sv[e / COLS][e % COLS] = rv[j];
    }
    if (SELECTIVE) {
      if (lane < CH) {
        const float dt = rb_softplus(rb + dt_bias);
        sb[lane] = dt;
        sg[0][lane] = expf(-rate * dt);
      }
    } else if (lane < CH) {
      sb[lane] = rb;
    }
    __syncthreads();
    if (t0 + CH < n) fetch(t0 + CH);                   // in flight while this chunk is computed
    __builtin_amdgcn_sched_barrier(0);                 // (issued here, not where the scheduler would sink them: at their use)
    // One token: with D = diag(g) S and u = beta (v - D^T k), the read-out of the updated state is
    // (D + k u^T)^T q = D^T q + u (k . q): one pass over the decayed column gives both dot products, and a token has
    // one reduction among the RG lanes on its way instead of two.  Two partial sums each: shorter chains of additions.
    auto token = [&](int tt) {
      const float vv = sv[tt][lane / RG];
      const float bt = sb[tt];
      const float gt = SELECTIVE ? sg[0][tt] : 0.f;
      float kv0 = 0.f, kv1 = 0.f, dq0 = 0.f, dq1 = 0.f, kq0 = 0.f, kq1 = 0.f;
#pragma unroll
      for (int i = 0; i < DKL; i += 2) {
        const float k0 = sk[tt][rg * DKL + i], q0 = sq[tt][rg * DKL + i];
        const float k1 = sk[tt][rg * DKL + i + 1], q1 = sq[tt][rg * DKL + i + 1];
        if (BONUS) {
          dq0 = fmaf(s[i], q0, dq0);
          dq1 = fmaf(s[i + 1], q1, dq1);
          kq0 = fmaf(ub[i] * k0, q0, kq0);
          kq1 = fmaf(ub[i + 1] * k1, q1, kq1);
          s[i] *= sg[tt][rg * DKL + i];
          s[i + 1] *= sg[tt][rg * DKL + i + 1];
          continue;
        }
        if (SELECTIVE) {
          s[i] *= gt;
          s[i + 1] *= gt;
          dq0 = fmaf(s[i], q0, dq0);
          dq1 = fmaf(s[i + 1], q1, dq1);
          kq0 = fmaf(k0, q0, kq0);
          kq1 = fmaf(k1, q1, kq1);
          continue;
        }
        s[i] *= sg[tt][rg * DKL + i];
        s[i + 1] *= sg[tt][rg * DKL + i + 1];
        kv0 = fmaf(s[i], k0, kv0);
        kv1 = fmaf(s[i + 1], k1, kv1);
        dq0 = fmaf(s[i], q0, dq0);
        dq1 = fmaf(s[i + 1], q1, dq1);
        kq0 = fmaf(k0, q0, kq0);
        kq1 = fmaf(k1, q1, kq1);
      }
      const float kv = (BONUS || SELECTIVE) ? 0.f : lanes_sum<RG>(kv0 + kv1);
      const float dq = lanes_sum<RG>(dq0 + dq1);
      const float kq = lanes_sum<RG>(kq0 + kq1);
      // without beta: the plain rule, S <- diag(g) S + k v^T
      const float u = SELECTIVE ? bt * vv : (!BONUS && beta) ? bt * (vv - kv) : vv;
#pragma unroll
      for (int i = 0; i < DKL; ++i) s[i] = fmaf(sk[tt][rg * DKL + i], u, s[i]);
      if (rg == 0) so[tt][lane / RG] = SELECTIVE ? fmaf(pass, vv, fmaf(u, kq, dq)) : fmaf(u, kq, dq);
    };
    if (nt == CH) {
      // a whole chunk as straight code, so that a token's reads from LDS are issued while the one before is computed
#pragma unroll
      for (int tt = 0; tt < CH; ++tt) token(tt);
    } else {
      for (int tt = 0; tt < nt; ++tt) token(tt);
    }
    __syncthreads();
    for (int e = lane; e < nt * COLS; e += RB_WAVE) {
      const int tt = e / COLS, c = e - tt * COLS;
      if (col0 + c < vdim) out[((size_t)(row0 + t0 + tt) * n_heads + h) * vdim + col0 + c] = so[tt][c];
    }
  }
  if (quads) {
#pragma unroll
    for (int i = 0; i < DKL; i += 4) {
      const int r = rg * DKL + i;
      if (on && r < dim) *reinterpret_cast<float4*>(S + r) = make_float4(s[i], s[i + 1], s[i + 2], s[i + 3]);
    }
  } else {
#pragma unroll
    for (int i = 0; i < DKL; ++i) {
      const int r = rg * DKL + i;
      if (on && r < dim) S[r] = s[i];
    }
  }
}

template <int DKL, int RG, int CH, int MODE>
static void launch_delta_rule(const float* q, const float* k, size_t qk_stride, const float* v, size_t v_stride,
                              const float* g, size_t g_stride, const float* beta, float* state, const int32_t* cu_seqlens,
                              const int32_t* slots, float* out, int n_seqs, int n_heads, int n_kv, int dim, int vdim,
                              int g_per_head, const float* bonus, const SelectiveArgs& sel, hipStream_t s) {
  constexpr int COLS = RB_WAVE / RG;
  static_assert((DKL * RG * CH) % RB_WAVE == 0 && CH <= RB_WAVE && DKL % 4 == 0, "a chunk's values are dealt evenly to the lanes");
  dim3 grid(n_seqs, n_heads, (vdim + COLS - 1) / COLS);
  delta_rule_kernel<DKL, RG, CH, MODE><<<grid, RB_WAVE, 0, s>>>(q, k, qk_stride, v, v_stride, g, g_stride, beta, state, cu_seqlens,
                                                                 slots, out, n_heads, n_kv, dim, vdim, g_per_head, bonus, sel);
}

extern "C" int rb_delta_rule(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                             const float* g, long long g_stride, const float* beta, float* state, const int32_t* cu_seqlens,
                             const int32_t* slots, float* out, int n_seqs, int n_tokens, int n_heads, int n_kv_heads, int dim,
                             int vdim, void* stream) {
  RB_RECORDED(rb_delta_rule(q, k, qk_stride, v, v_stride, g, g_stride, beta, state, cu_seqlens, slots, out, n_seqs, n_tokens,
                            n_heads, n_kv_heads, dim, vdim, stream));
  RB_REQUIRE(beta != nullptr, "rb_delta_rule: the delta rule needs beta");
  return rb_linear_recurrence(q, k, qk_stride, v, v_stride, g, g_stride, 0, beta, state, cu_seqlens, slots, out, n_seqs, n_tokens,
                              n_heads, n_kv_heads, dim, vdim, stream);
}

extern "C" int rb_linear_recurrence(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                                    const float* g, long long g_stride, int g_per_head, const float* beta, float* state,
                                    const int32_t* cu_seqlens, const int32_t* slots, float* out, int n_seqs, int n_tokens,
                                    int n_heads, int n_kv_heads, int dim, int vdim, void* stream) {
  RB_RECORDED(rb_linear_recurrence(q, k, qk_stride, v, v_stride, g, g_stride, g_per_head, beta, state, cu_seqlens, slots, out, n_seqs,
                                   n_tokens, n_heads, n_kv_heads, dim, vdim, stream));
  return rb_linear_recurrence_bonus(q, k, qk_stride, v, v_stride, g, g_stride, g_per_head, beta, nullptr, state, cu_seqlens, slots,
                                    out, n_seqs, n_tokens, n_heads, n_kv_heads, dim, vdim, stream);
}

static int linear_recurrence_launch(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                                    const float* g, long long g_stride, int g_per_head, const float* beta, const float* bonus,
                                    int silu_in, float* state, const int32_t* cu_seqlens, const int32_t* slots, float* out, int n_seqs,
                                    int n_tokens, int n_heads, int n_kv_heads, int dim, int vdim, const SelectiveArgs* sel, void* stream);

// bonus (float32 [H, dim], null: rb_linear_recurrence): the plain rule read BEFORE the token's write, with the token's own
// k v^T weighted per key channel:  out = (S + diag(bonus) k v^T)^T q;  S <- diag(g) S + k v^T.  Goes without beta.
extern "C" int rb_linear_recurrence_bonus(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                                          const float* g, long long g_stride, int g_per_head, const float* beta,
                                          const float* bonus, float* state, const int32_t* cu_seqlens, const int32_t* slots,
                                          float* out, int n_seqs, int n_tokens, int n_heads, int n_kv_heads, int dim, int vdim,
                                          void* stream) {
  RB_RECORDED(rb_linear_recurrence_bonus(q, k, qk_stride, v, v_stride, g, g_stride, g_per_head, beta, bonus, state, cu_seqlens, slots,
                                         out, n_seqs, n_tokens, n_heads, n_kv_heads, dim, vdim, stream));
  return linear_recurrence_launch(q, k, qk_stride, v, v_stride, g, g_stride, g_per_head, beta, bonus, 0, state, cu_seqlens, slots, out,
                                  n_seqs, n_tokens, n_heads, n_kv_heads, dim, vdim, nullptr, stream);
}

// The plain rule with one constant decay per head (decay float32 [H]) and silu on q, k and v as they are read:
// S <- decay[h] S + k v^T, out = S^T q, token after token.  q and k have as many heads as v.
extern "C" int rb_lightning_recurrence(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                                       const float* decay, float* state, const int32_t* cu_seqlens, const int32_t* slots, float* out,
                                       int n_seqs, int n_tokens, int n_heads, int dim, int vdim, void* stream) {
  RB_RECORDED(rb_lightning_recurrence(q, k, qk_stride, v, v_stride, decay, state, cu_seqlens, slots, out, n_seqs, n_tokens, n_heads, dim,
                                      vdim, stream));
  return linear_recurrence_launch(q, k, qk_stride, v, v_stride, decay, 0, 1, nullptr, nullptr, 1, state, cu_seqlens, slots, out, n_seqs,
                                  n_tokens, n_heads, n_heads, dim, vdim, nullptr, stream);
}

// A selective scan, token after token: with dt = softplus(dt_in[t * dt_stride + h] + dt_bias[h]),
//   S <- exp(-exp(a_log[h]) dt) S + dt k v^T;  out[t, h, :] = S^T q + d[h] v      (head h reads the q and k of group h / (H / G))
extern "C" int rb_selective_scan(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride, const float* dt_in,
                                 long long dt_stride, const float* dt_bias, const float* a_log, const float* d, float* state,
                                 const int32_t* cu_seqlens, const int32_t* slots, float* out, int n_seqs, int n_tokens, int n_heads,
                                 int n_groups, int dim, int vdim, void* stream) {
  RB_RECORDED(rb_selective_scan(q, k, qk_stride, v, v_stride, dt_in, dt_stride, dt_bias, a_log, d, state, cu_seqlens, slots, out, n_seqs,
                                n_tokens, n_heads, n_groups, dim, vdim, stream));
  RB_REQUIRE(dt_stride >= n_heads && dt_in != nullptr && dt_bias != nullptr && a_log != nullptr && d != nullptr,
             "rb_selective_scan: the step sizes' rows are too short, or a tensor is missing");
  const SelectiveArgs sel = {dt_in, (size_t)dt_stride, dt_bias, a_log, d};
  return linear_recurrence_launch(q, k, qk_stride, v, v_stride, nullptr, n_heads, 1, nullptr, nullptr, 0, state, cu_seqlens, slots, out,
                                  n_seqs, n_tokens, n_heads, n_groups, dim, vdim, &sel, stream);
}

// silu_in: q, k and v go through silu as they are read; g_stride 0 (with g_per_head): the same decays for every token.
static int linear_recurrence_launch(const float* q, const float* k, long long qk_stride, const float* v, long long v_stride,
                                    const float* g, long long g_stride, int g_per_head, const float* beta, const float* bonus,
                                    int silu_in, float* state, const int32_t* cu_seqlens, const int32_t* slots, float* out, int n_seqs,
                                    int n_tokens, int n_heads, int n_kv_heads, int dim, int vdim, const SelectiveArgs* selective,
                                    void* stream) {
  const SelectiveArgs sel = selective ? *selective : SelectiveArgs{nullptr, 0, nullptr, nullptr, nullptr};
  RB_REQUIRE(bonus == nullptr || beta == nullptr, "rb_linear_recurrence: a bonus goes with the plain rule (no beta)");
  RB_REQUIRE(n_seqs >= 0 && n_heads > 0 && n_kv_heads > 0 && n_heads % n_kv_heads == 0 && dim > 0 && vdim > 0,
             "rb_linear_recurrence: bad sizes H=%d Hk=%d dim=%d vdim=%d", n_heads, n_kv_heads, dim, vdim);
  RB_REQUIRE((g_stride == 0 && g_per_head && silu_in) || g_stride >= (long long)n_heads * (g_per_head ? 1 : dim),
             "rb_linear_recurrence: the decays' row stride is too short");
  RB_REQUIRE(dim <= 512, "rb_linear_recurrence: key size %d not supported (at most 512)", dim);
  RB_REQUIRE(n_heads <= 65535 && vdim <= 65535 * 4, "rb_linear_recurrence: too many heads or value channels");
  if (n_seqs == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const size_t qs = (size_t)qk_stride, vs = (size_t)v_stride;
  // a step of one token per sequence (n_tokens == n_seqs) stages chunks of as few tokens as deal evenly to the lanes:
  // the machinery of a chunk of 16 would cost it several times its arithmetic
  const bool single = n_tokens <= n_seqs;
#define DR_GO(DKL, RG, CH)                                                                                                  \
  do {                                                                                                                      \
    constexpr int CH1 = (DKL * RG >= RB_WAVE) ? 1 : RB_WAVE / (DKL * RG);                                                   \
    if (single && selective)                                                                                                \
      launch_delta_rule<DKL, RG, CH1, 3>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,        \
                                         n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                \
    else if (selective)                                                                                                     \
      launch_delta_rule<DKL, RG, CH, 3>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,         \
                                        n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                 \
    else if (single && silu_in)                                                                                                  \
      launch_delta_rule<DKL, RG, CH1, 2>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,        \
                                         n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                   \
    else if (silu_in)                                                                                                       \
      launch_delta_rule<DKL, RG, CH, 2>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,         \
                                        n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                    \
    else if (single && bonus)                                                                                               \
      launch_delta_rule<DKL, RG, CH1, 1>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,     \
                                            n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                \
    else if (single)                                                                                                        \
      launch_delta_rule<DKL, RG, CH1, 0>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,    \
                                             n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);               \
    else if (bonus)                                                                                                         \
      launch_delta_rule<DKL, RG, CH, 1>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,      \
                                           n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                 \
    else                                                                                                                    \
      launch_delta_rule<DKL, RG, CH, 0>(q, k, qs, v, vs, g, (size_t)g_stride, beta, state, cu_seqlens, slots, out,     \
                                            n_seqs, n_heads, n_kv_heads, dim, vdim, g_per_head, bonus, sel, s);                \
  } while (0)
  // Rows of a column over RG lanes, chunks as long as the registers that hold the next one allow.  A token's time is
  // its lane's share of the column, so while the waves do not fill the GPU's SIMDs a column goes to more lanes
  // (more and shorter waves); once they do, fewer lanes per column save the moves between them.
  const long long simds = 4LL * rb_compute_units();
  auto waves = [&](int rg) { return (long long)n_seqs * n_heads * ((vdim + RB_WAVE / rg - 1) / (RB_WAVE / rg)); };
  if (dim <= 16)
    DR_GO(4, 4, 16);
  else if (dim <= 32) {
    if (waves(4) >= simds) DR_GO(8, 4, 16);
    else DR_GO(4, 8, 16);
  } else if (dim <= 64) {
    if (waves(8) >= simds) DR_GO(8, 8, 16);
    else DR_GO(4, 16, 16);
  } else if (dim <= 128) {
    if (waves(8) >= simds) DR_GO(16, 8, 16);
    else DR_GO(8, 16, 16);
  } else if (dim <= 256)
    DR_GO(16, 16, 8);
  else
    DR_GO(32, 16, 4);
#undef DR_GO
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- read-out norm with gate
// out[t, h, :] = o[t, h, :] / sqrt(mean(o^2) + eps) * weight * sigmoid(gate[t, h, :]); a wave per (token, head).
template <typename TO>
__global__ void gated_rmsnorm_kernel(const float* __restrict__ o, const float* __restrict__ weight,
                                     const float* __restrict__ gate, size_t gate_stride, float eps, TO* __restrict__ out,
                                     int n_heads, int vdim, long long n_pairs, int act, size_t weight_head_stride) {
  const long long pair = (long long)blockIdx.x * (blockDim.x / RB_WAVE) + threadIdx.x / RB_WAVE;
  if (pair >= n_pairs) return;
  const int lane = threadIdx.x & (RB_WAVE - 1);
  const size_t t = (size_t)(pair / n_heads);
  const int h = (int)(pair % n_heads);
  const float* p = o + (size_t)pair * vdim;
  const float* gp = gate + t * gate_stride + (size_t)h * vdim;
  const float* wp = weight + (size_t)h * weight_head_stride;
  float ss = 0.f;
  for (int i = lane; i < vdim; i += RB_WAVE) ss = fmaf(p[i], p[i], ss);
  ss = wave_sum(ss);
  const float f = 1.0f / sqrtf(ss / (float)vdim + eps);
  for (int i = lane; i < vdim; i += RB_WAVE)
    Num<TO>::store(out + (size_t)pair * vdim + i, p[i] * f * wp[i] * (act == 1 ? gp[i] * rb_sigmoid(gp[i]) : rb_sigmoid(gp[i])));
}

// The same for rows of many numbers (one norm over all heads together): a workgroup a row, 16-byte accesses where they fit.
template <typename TO, bool VEC>
__global__ __launch_bounds__(1024) void gated_rmsnorm_row_kernel(const float* __restrict__ o, const float* __restrict__ weight,
                                                                 const float* __restrict__ gate, size_t gate_stride, float eps,
                                                                 TO* __restrict__ out, int width, int act) {
  __shared__ float scratch[16];
  const size_t t = blockIdx.x;
  const float* p = o + t * width;
  const float* gp = gate + t * gate_stride;
  auto gated = [&](float g) { return act == 1 ? g * rb_sigmoid(g) : rb_sigmoid(g); };
  float ss = 0.f;
  if (VEC) {
    const int j0 = 4 * threadIdx.x;
    float4 keep = make_float4(0.f, 0.f, 0.f, 0.f), g0 = keep;
    for (int j = j0; j < width; j += 4 * blockDim.x) {
      const float4 v = *reinterpret_cast<const float4*>(p + j);
      if (j == j0) {
        keep = v;
        g0 = *reinterpret_cast<const float4*>(gp + j);
      }
      ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    }
    const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
    for (int j = j0; j < width; j += 4 * blockDim.x) {
      const float4 v = j == j0 ? keep : *reinterpret_cast<const float4*>(p + j);
      const float4 g = j == j0 ? g0 : *reinterpret_cast<const float4*>(gp + j);
      const float4 w = *reinterpret_cast<const float4*>(weight + j);
      const float a = v.x * f * w.x * gated(g.x), b = v.y * f * w.y * gated(g.y), c = v.z * f * w.z * gated(g.z),
                  d = v.w * f * w.w * gated(g.w);
      if (sizeof(TO) == 4)
        *reinterpret_cast<float4*>(out + t * width + j) = make_float4(a, b, c, d);
      else
        *reinterpret_cast<uint2*>(out + t * width + j) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
    }
  } else {
    for (int j = threadIdx.x; j < width; j += blockDim.x) ss = fmaf(p[j], p[j], ss);
    const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
    for (int j = threadIdx.x; j < width; j += blockDim.x) Num<TO>::store(out + t * width + j, p[j] * f * weight[j] * gated(gp[j]));
  }
}

// out[t, :] = o[t, :] / sqrt(mean(o[t, :]^2) + eps) * weight * act(gate[t, :]) over the whole row (act 0: sigmoid, 1: silu).
extern "C" int rb_gated_rmsnorm_rows(const float* o, const float* weight, const float* gate, long long gate_stride, int act, float eps,
                                     void* out, int out_dtype, int n_tokens, int width, void* stream) {
  RB_RECORDED(rb_gated_rmsnorm_rows(o, weight, gate, gate_stride, act, eps, out, out_dtype, n_tokens, width, stream));
  RB_REQUIRE(n_tokens >= 0 && width > 0 && (act == 0 || act == 1) && gate_stride >= width, "rb_gated_rmsnorm_rows: bad sizes");
  RB_REQUIRE(out_dtype == RB_F32 || out_dtype == RB_BF16, "rb_gated_rmsnorm_rows: unknown dtype %d", out_dtype);
  if (n_tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool vec = width % 4 == 0 && gate_stride % 4 == 0 && aligned(o) && aligned(weight) && aligned(gate) && aligned(out);
  int threads = ((width / (vec ? 4 : 1) + RB_WAVE - 1) / RB_WAVE) * RB_WAVE;
  threads = threads > 1024 ? 1024 : (threads < RB_WAVE ? RB_WAVE : threads);
#define RB_GR(TO, VEC) \
  gated_rmsnorm_row_kernel<TO, VEC><<<n_tokens, threads, 0, s>>>(o, weight, gate, (size_t)gate_stride, eps, (TO*)out, width, act)
  if (out_dtype == RB_F32) {
    if (vec) RB_GR(float, true);
    else RB_GR(float, false);
  } else {
    if (vec) RB_GR(bf16_t, true);
    else RB_GR(bf16_t, false);
  }
#undef RB_GR
  RB_LAUNCH_CHECK();
  return 0;
}

// The gate in front of the norm, and the row in equal parts with a norm each: with g = o * silu(gate),
//   out[t, part] = g[part] / sqrt(mean(g[part]^2) + eps) * weight[part].      A workgroup a token and part.
template <typename TO, bool VEC>
__global__ __launch_bounds__(1024) void gate_rmsnorm_parts_kernel(const float* __restrict__ o, const float* __restrict__ weight,
                                                                  const float* __restrict__ gate, size_t gate_stride, float eps,
                                                                  TO* __restrict__ out, int width, int part) {
  __shared__ float scratch[16];
  const size_t t = blockIdx.x;
  const int c0 = blockIdx.y * part;
  const float* p = o + t * width + c0;
  const float* gp = gate + t * gate_stride + c0;
  const float* wp = weight + c0;
  TO* op = out + t * width + c0;
  auto gated = [](float v, float g) { return v * g * rb_sigmoid(g); };
  float ss = 0.f;
  if (VEC) {
    const int j0 = 4 * threadIdx.x;
    auto quad = [&](int j) {
      const float4 v = *reinterpret_cast<const float4*>(p + j), g = *reinterpret_cast<const float4*>(gp + j);
      return make_float4(gated(v.x, g.x), gated(v.y, g.y), gated(v.z, g.z), gated(v.w, g.w));
    };
    float4 keep = make_float4(0.f, 0.f, 0.f, 0.f), w0 = keep;
    for (int j = j0; j < part; j += 4 * blockDim.x) {
      const float4 v = quad(j);
      if (j == j0) {
        keep = v;
        w0 = *reinterpret_cast<const float4*>(wp + j);
      }
      ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
    }
    const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)part + eps);
    for (int j = j0; j < part; j += 4 * blockDim.x) {
      const float4 v = j == j0 ? keep : quad(j);
      const float4 w = j == j0 ? w0 : *reinterpret_cast<const float4*>(wp + j);
      const float a = v.x * f * w.x, b = v.y * f * w.y, c = v.z * f * w.z, d = v.w * f * w.w;
      if (sizeof(TO) == 4)
        *reinterpret_cast<float4*>(op + j) = make_float4(a, b, c, d);
      else
        *reinterpret_cast<uint2*>(op + j) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
    }
  } else {
    for (int j = threadIdx.x; j < part; j += blockDim.x) {
      const float v = gated(p[j], gp[j]);
      ss = fmaf(v, v, ss);
    }
    const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)part + eps);
    for (int j = threadIdx.x; j < part; j += blockDim.x) Num<TO>::store(op + j, gated(p[j], gp[j]) * f * wp[j]);
  }
}

extern "C" int rb_gate_rmsnorm_parts(const float* o, const float* weight, const float* gate, long long gate_stride, float eps, void* out,
                                     int out_dtype, int n_tokens, int width, int parts, void* stream) {
  RB_RECORDED(rb_gate_rmsnorm_parts(o, weight, gate, gate_stride, eps, out, out_dtype, n_tokens, width, parts, stream));
  RB_REQUIRE(n_tokens >= 0 && width > 0 && parts > 0 && parts <= 65535 && width % parts == 0 && gate_stride >= width,
             "rb_gate_rmsnorm_parts: bad sizes T=%d width=%d parts=%d", n_tokens, width, parts);
  RB_REQUIRE(out_dtype == RB_F32 || out_dtype == RB_BF16, "rb_gate_rmsnorm_parts: unknown dtype %d", out_dtype);
  if (n_tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const int part = width / parts;
  const bool vec = part % 4 == 0 && gate_stride % 4 == 0 && aligned(o) && aligned(weight) && aligned(gate) && aligned(out);
  int threads = ((part / (vec ? 4 : 1) + RB_WAVE - 1) / RB_WAVE) * RB_WAVE;
  threads = threads > 1024 ? 1024 : (threads < RB_WAVE ? RB_WAVE : threads);
  const dim3 grid(n_tokens, parts);
#define RB_GP(TO, VEC) \
  gate_rmsnorm_parts_kernel<TO, VEC><<<grid, threads, 0, s>>>(o, weight, gate, (size_t)gate_stride, eps, (TO*)out, width, part)
  if (out_dtype == RB_F32) {
    if (vec) RB_GP(float, true);
    else RB_GP(float, false);
  } else {
    if (vec) RB_GP(bf16_t, true);
    else RB_GP(bf16_t, false);
  }
#undef RB_GP
  RB_LAUNCH_CHECK();
  return 0;
}

extern "C" int rb_gated_rmsnorm(const float* o, const float* weight, const float* gate, long long gate_stride, float eps,
                                void* out, int out_dtype, int n_tokens, int n_heads, int vdim, void* stream) {
  RB_RECORDED(rb_gated_rmsnorm(o, weight, gate, gate_stride, eps, out, out_dtype, n_tokens, n_heads, vdim, stream));
  return rb_gated_rmsnorm_act(o, weight, gate, gate_stride, 0, eps, out, out_dtype, n_tokens, n_heads, vdim, stream);
}

// act 0: the gate is sigmoid(gate); 1: silu(gate) = gate * sigmoid(gate)
extern "C" int rb_gated_rmsnorm_act(const float* o, const float* weight, const float* gate, long long gate_stride, int act, float eps,
                                    void* out, int out_dtype, int n_tokens, int n_heads, int vdim, void* stream) {
  RB_RECORDED(rb_gated_rmsnorm_act(o, weight, gate, gate_stride, act, eps, out, out_dtype, n_tokens, n_heads, vdim, stream));
  return rb_gated_rmsnorm_heads(o, weight, 0, gate, gate_stride, act, eps, out, out_dtype, n_tokens, n_heads, vdim, stream);
}

// The same with head h's weight at weight + h * weight_head_stride (0: one weight of vdim numbers for all heads; vdim: a
// weight over the concatenated heads).
extern "C" int rb_gated_rmsnorm_heads(const float* o, const float* weight, long long weight_head_stride, const float* gate,
                                      long long gate_stride, int act, float eps, void* out, int out_dtype, int n_tokens, int n_heads,
                                      int vdim, void* stream) {
  RB_RECORDED(rb_gated_rmsnorm_heads(o, weight, weight_head_stride, gate, gate_stride, act, eps, out, out_dtype, n_tokens, n_heads,
                                     vdim, stream));
  RB_REQUIRE(weight_head_stride >= 0, "rb_gated_rmsnorm: bad weight stride");
  RB_REQUIRE(n_tokens >= 0 && n_heads > 0 && vdim > 0 && (act == 0 || act == 1), "rb_gated_rmsnorm: bad sizes");
  RB_REQUIRE(gate_stride >= (long long)n_heads * vdim, "rb_gated_rmsnorm: the gate's row stride is too short");
  if (n_tokens == 0) return 0;
  const long long n_pairs = (long long)n_tokens * n_heads;
  const int grid = (int)((n_pairs + 3) / 4);
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == RB_F32)
    gated_rmsnorm_kernel<float><<<grid, 256, 0, s>>>(o, weight, gate, (size_t)gate_stride, eps, (float*)out, n_heads, vdim, n_pairs, act,
                                                     (size_t)weight_head_stride);
  else if (out_dtype == RB_BF16)
    gated_rmsnorm_kernel<bf16_t><<<grid, 256, 0, s>>>(o, weight, gate, (size_t)gate_stride, eps, (bf16_t*)out, n_heads, vdim, n_pairs, act,
                                                      (size_t)weight_head_stride);
  else
    RB_REQUIRE(false, "rb_gated_rmsnorm: unknown dtype %d", out_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}
