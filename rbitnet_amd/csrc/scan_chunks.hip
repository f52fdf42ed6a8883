// A selective scan (rb_selective_scan) for steps that bring many tokens of a sequence, in chunks of 128 tokens on the matrix cores.
// Per head, with a_t = exp(a_log) dt_t log2(e), c_t = - sum of a over the chunk up to t (so that 2^(c_i - c_j) is the decay from
// token j to token i), S the state in front of the chunk and L its last token:
//   y_i = sum_(j <= i) dt_j 2^(c_i - c_j) (q_i . k_j) x_j  +  2^(c_i) S^T q_i  +  d x_i
//   S'  = 2^(c_L) S + sum_j k_j (dt_j 2^(c_L - c_j) x_j)^T
// Three launches, of which only the second goes from chunk to chunk, and only element by element:
//   1. what every chunk adds to the state (a workgroup a chunk and head);
//   2. the state in front of every chunk, and behind the last one (a thread eight elements of a head's state);
//   3. the outputs (a workgroup a chunk and head).
// q, k and x are bfloat16 (they come out of a convolution that may be so stored); decays, step sizes, sums and the state are
// float32.  Where a float32 number meets the matrix cores as an operand that the state depends on, it goes in as two bfloat16
// numbers, the rounded one and what is left of it: the step-size-weighted x of launch 1, and the state in launch 3.  The weights of
// a chunk's own tokens, which reach the output alone, are rounded once, as attention's are.
// Chunks are counted from the start of a sequence's piece of the step.
#include <math.h>

#include "api.h"
#include "common.h"
#include "mfma.h"

#define SK_CHUNK 128
#define SK_MAX_DIM 256
#define SK_MAX_VDIM 128

struct ScanArgs {
  const bf16_t *x, *k, *q;
  size_t stride;
  const float* dt_in;
  size_t dt_stride;
  const float *dt_bias, *a_log, *d;
  float* state;
  const int32_t *cu, *slots;
  float* out;
  float* added;          // [chunks][H][VP / 16][NP / 32][64][8]: what a chunk adds to the state, in the matrix cores' order
  bf16_t* before;        // [chunks][H][VP / 16][NP / 32][2][64][8]: the state in front of a chunk, rounded, and the rest
  float* total;          // [chunks][H]: c_L
  int n_seqs, n_heads, n_groups, dim, vdim, n_chunks;
};

// The chunk `at` of the step: sequences one after the other, each with as many chunks as its piece fills.
__device__ __forceinline__ bool sk_find(const ScanArgs& p, int at, int& row0, int& len) {
  for (int b = 0; b < p.n_seqs; ++b) {
    const int n = p.cu[b + 1] - p.cu[b], chunks = (n + SK_CHUNK - 1) / SK_CHUNK;
    if (at < chunks) {
      row0 = p.cu[b] + at * SK_CHUNK;
      len = n - at * SK_CHUNK < SK_CHUNK ? n - at * SK_CHUNK : SK_CHUNK;
      return true;
    }
    at -= chunks;
  }
  return false;
}

// Workgroups are dealt to the 8 XCDs in turn: each XCD gets neighbouring (chunk, head) pairs, whose heads share q and k.
__device__ __forceinline__ bool sk_item(const ScanArgs& p, int& chunk, int& h) {
  const int work = p.n_chunks * p.n_heads, per = (work + 7) / 8;
  const int item = (blockIdx.x % 8) * per + blockIdx.x / 8;
  if (blockIdx.x / 8 >= per || item >= work) return false;
  chunk = item / p.n_heads;
  h = item - chunk * p.n_heads;
  return true;
}

__device__ __forceinline__ float sk_softplus(float v) { return v > 20.0f ? v : log1pf(expf(v)); }

// Step sizes and running decays of the chunk's tokens, by the first 128 threads; tokens past its end have steps of zero.
__device__ __forceinline__ void sk_steps(const ScanArgs& p, int h, int row0, int len, float* cl, float* dts, float* carry) {
  const int tid = threadIdx.x, lane = tid & (RB_WAVE - 1);
  float dt = 0.f, c = 0.f;
  if (tid < SK_CHUNK) {
    if (tid < len) dt = sk_softplus(p.dt_in[(size_t)(row0 + tid) * p.dt_stride + h] + p.dt_bias[h]);
    c = -expf(p.a_log[h]) * dt * 1.44269504088896341f;
#pragma unroll
    for (int o = 1; o < RB_WAVE; o <<= 1) {
      const float up = __shfl_up(c, o, RB_WAVE);
      if (lane >= o) c += up;
    }
    if (tid == RB_WAVE - 1) *carry = c;
  }
  __syncthreads();
  if (tid < SK_CHUNK) {
    cl[tid] = tid >= RB_WAVE ? c + *carry : c;
    dts[tid] = dt;
  }
  __syncthreads();
}

typedef __attribute__((ext_vector_type(4))) short sk_i16x4_t;
__device__ __forceinline__ uint2 sk_read_transposed(const uint16_t* p) {
  union {
    sk_i16x4_t v;
    uint2 u;
  } r;
  r.v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) sk_i16x4_t*)(p));
  return r.u;
}
// An operand whose depth are tokens, from rows of tokens in LDS: lane l gets channel col0 + l % 16 of tokens
// tok0 + 4 (l / 16) + 0..3 and the same 16 tokens further on.
__device__ __forceinline__ Frag8 sk_tokens_frag(const uint16_t* rows, int ld, int tok0, int col0) {
  const int lane = threadIdx.x & (RB_WAVE - 1), s = lane & 15, g = lane >> 4;
  const uint16_t* p = rows + (tok0 + 4 * g + (s >> 2)) * ld + col0 + 4 * (s & 3);
  const uint2 a = sk_read_transposed(p), b = sk_read_transposed(p + 16 * ld);
  Frag8 f;
  f.u = make_uint4(a.x, a.y, b.x, b.y);
  return f;
}

// ---------------------------------------------------------------- 1: what a chunk adds to the state
// KN: dim rounded up to 32 KN; VT: vdim rounded up to 16 VT (zeros beyond).  The state's rows are the product's rows.
template <int KN, int VT>
__global__ __launch_bounds__(256) void scan_added_kernel(ScanArgs p) {
  constexpr int NP = 32 * KN, VP = 16 * VT, KLD = NP + 16, XLD = VP + 16;
  constexpr int WN = 2 * KN < 4 ? 2 * KN : 4, WV = 4 / WN;       // the four waves over row tiles and column tiles
  constexpr int NT = 2 * KN / WN, VW = VT / WV;
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  uint16_t* ks = lds;                                  // [128][KLD]
  uint16_t* xh = ks + SK_CHUNK * KLD;                  // [128][XLD]: weighted x, rounded
  uint16_t* xl = xh + SK_CHUNK * XLD;                  //             and the rest
  __shared__ float cl[SK_CHUNK], dts[SK_CHUNK], carry;
  int chunk, h, row0, len;
  if (!sk_item(p, chunk, h) || !sk_find(p, chunk, row0, len)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4;
  const bf16_t* kp = p.k + (size_t)row0 * p.stride + (size_t)(h / (p.n_heads / p.n_groups)) * p.dim;
  const bf16_t* xp = p.x + (size_t)row0 * p.stride + (size_t)h * p.vdim;
  const int n_tok = (len + 31) / 32 * 32;
  for (int e = tid; e < n_tok * (NP / 8); e += 256) {
    const int j = e / (NP / 8), c = 8 * (e - j * (NP / 8));
    *reinterpret_cast<uint4*>(ks + j * KLD + c) = (j < len && c < p.dim) ? load16(kp + (size_t)j * p.stride + c) : zero16();
  }
  sk_steps(p, h, row0, len, cl, dts, &carry);
  const float c_last = cl[len - 1];
  if (tid == 0) p.total[(size_t)chunk * p.n_heads + h] = c_last;
  for (int e = tid; e < n_tok * (VP / 8); e += 256) {
    const int j = e / (VP / 8), c = 8 * (e - j * (VP / 8));
    uint4 hi = zero16(), lo = zero16();
    if (j < len && c < p.vdim) {
      const uint4 raw = load16(xp + (size_t)j * p.stride + c);
      const float w = dts[j] * __builtin_amdgcn_exp2f(c_last - cl[j]);
      auto split = [&](uint32_t two, uint32_t& a, uint32_t& b) {
        const float u = bf16_bits_to_f32(two & 0xffffu) * w, v = bf16_bits_to_f32(two >> 16) * w;
        a = pack_bf16x2(u, v);
        b = pack_bf16x2(u - bf16_bits_to_f32(a & 0xffffu), v - bf16_bits_to_f32(a >> 16));
      };
      split(raw.x, hi.x, lo.x);
      split(raw.y, hi.y, lo.y);
      split(raw.z, hi.z, lo.z);
      split(raw.w, hi.w, lo.w);
    }
    *reinterpret_cast<uint4*>(xh + j * XLD + c) = hi;
    *reinterpret_cast<uint4*>(xl + j * XLD + c) = lo;
  }
  __syncthreads();
  const int nt0 = (wave % WN) * NT, vt0 = (wave / WN) * VW;
  f32x4_t acc[NT][VW];
#pragma unroll
  for (int a = 0; a < NT; ++a)
#pragma unroll
    for (int b = 0; b < VW; ++b) acc[a][b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int t0 = 0; t0 < n_tok; t0 += 32) {
    Frag8 kf[NT];
#pragma unroll
    for (int a = 0; a < NT; ++a) kf[a] = sk_tokens_frag(ks, KLD, t0, 16 * (nt0 + a));
#pragma unroll
    for (int b = 0; b < VW; ++b) {
      const Frag8 hi = sk_tokens_frag(xh, XLD, t0, 16 * (vt0 + b)), lo = sk_tokens_frag(xl, XLD, t0, 16 * (vt0 + b));
#pragma unroll
      for (int a = 0; a < NT; ++a) acc[a][b] = mfma16(kf[a], lo, acc[a][b]);
#pragma unroll
      for (int a = 0; a < NT; ++a) acc[a][b] = mfma16(kf[a], hi, acc[a][b]);
    }
  }
  // row 16 nt + 4 g + i of the state, column 16 vt + l % 16
  float* dst = p.added + ((size_t)chunk * p.n_heads + h) * (NP * VP);
#pragma unroll
  for (int a = 0; a < NT; ++a) {
    const int n = 16 * (nt0 + a) + 4 * g;
#pragma unroll
    for (int b = 0; b < VW; ++b) {
      float* q = dst + ((size_t)(vt0 + b) * KN + n / 32) * 512 + ((lane & 15) + 16 * ((n % 32) / 8)) * 8 + n % 8;
      *reinterpret_cast<float4*>(q) = make_float4(acc[a][b][0], acc[a][b][1], acc[a][b][2], acc[a][b][3]);
    }
  }
}

// ---------------------------------------------------------------- 2: from chunk to chunk
template <int KN, int VT>
__global__ __launch_bounds__(256) void scan_carry_kernel(ScanArgs p) {
  constexpr int NP = 32 * KN, VP = 16 * VT, AHEAD = 4;
  const int e = blockIdx.z * 256 + threadIdx.x;
  if (e >= NP * VP / 8) return;
  const int b = blockIdx.x, h = blockIdx.y;
  int first = 0;
  for (int i = 0; i < b; ++i) first += (p.cu[i + 1] - p.cu[i] + SK_CHUNK - 1) / SK_CHUNK;
  const int n_tok = p.cu[b + 1] - p.cu[b], chunks = (n_tok + SK_CHUNK - 1) / SK_CHUNK;
  if (chunks <= 0) return;
  const int block = e / 64, l = e % 64;
  const int v = 16 * (block / KN) + (l & 15), n = 32 * (block % KN) + 8 * (l >> 4);
  const bool on = v < p.vdim && n < p.dim;
  float* S = p.state + (((size_t)p.slots[b] * p.n_heads + h) * p.vdim + (on ? v : 0)) * p.dim + (on ? n : 0);
  float s[8];
  {
    const float4 a = on ? *reinterpret_cast<const float4*>(S) : make_float4(0.f, 0.f, 0.f, 0.f);
    const float4 c = on ? *reinterpret_cast<const float4*>(S + 4) : make_float4(0.f, 0.f, 0.f, 0.f);
    s[0] = a.x, s[1] = a.y, s[2] = a.z, s[3] = a.w, s[4] = c.x, s[5] = c.y, s[6] = c.z, s[7] = c.w;
  }
  const size_t step = (size_t)p.n_heads * (NP * VP);
  const float* src = p.added + ((size_t)first * p.n_heads + h) * (NP * VP) + (size_t)e * 8;
  bf16_t* dst = p.before + 2 * (((size_t)first * p.n_heads + h) * (NP * VP)) + (size_t)block * 1024 + l * 8;
  const float* tot = p.total + (size_t)first * p.n_heads + h;
  for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
    float4 a[AHEAD], c[AHEAD];
    float t[AHEAD];
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      const int at = c0 + u < chunks ? c0 + u : chunks - 1;
      a[u] = *reinterpret_cast<const float4*>(src + at * step);
      c[u] = *reinterpret_cast<const float4*>(src + at * step + 4);
      t[u] = tot[(size_t)at * p.n_heads];
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < AHEAD; ++u) {
      if (c0 + u >= chunks) break;
      uint4 hi, lo;
      auto split = [](float x, float y, uint32_t& r, uint32_t& rest) {
        r = pack_bf16x2(x, y);
        rest = pack_bf16x2(x - bf16_bits_to_f32(r & 0xffffu), y - bf16_bits_to_f32(r >> 16));
      };
      split(s[0], s[1], hi.x, lo.x);
      split(s[2], s[3], hi.y, lo.y);
      split(s[4], s[5], hi.z, lo.z);
      split(s[6], s[7], hi.w, lo.w);
      bf16_t* q = dst + 2 * (size_t)(c0 + u) * step;
      *reinterpret_cast<uint4*>(q) = hi;
      *reinterpret_cast<uint4*>(q + 512) = lo;
      const float f = __builtin_amdgcn_exp2f(t[u]);
      s[0] = fmaf(f, s[0], a[u].x), s[1] = fmaf(f, s[1], a[u].y), s[2] = fmaf(f, s[2], a[u].z), s[3] = fmaf(f, s[3], a[u].w);
      s[4] = fmaf(f, s[4], c[u].x), s[5] = fmaf(f, s[5], c[u].y), s[6] = fmaf(f, s[6], c[u].z), s[7] = fmaf(f, s[7], c[u].w);
    }
  }
  if (on) {
    *reinterpret_cast<float4*>(S) = make_float4(s[0], s[1], s[2], s[3]);
    *reinterpret_cast<float4*>(S + 4) = make_float4(s[4], s[5], s[6], s[7]);
  }
}

// ---------------------------------------------------------------- 3: the outputs
// Wave w takes queries 16 w .. and 16 (7 - w) .. of the chunk: scores transposed (keys x queries), so that they leave the first
// product in the layout that the second wants; the outputs transposed too (value channels x queries), so that what belongs to
// a query is one number a lane.
template <int KN, int VT>
__global__ __launch_bounds__(256) void scan_outputs_kernel(ScanArgs p) {
  constexpr int NP = 32 * KN, VP = 16 * VT, KLD = NP + 8, XLD = VP + 16;
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  uint16_t* ks = lds;                                  // [128][KLD]
  uint16_t* xs = ks + SK_CHUNK * KLD;                  // [128][XLD]
  __shared__ __attribute__((aligned(16))) float cl[SK_CHUNK], dts[SK_CHUNK];
  __shared__ float carry;
  int chunk, h, row0, len;
  if (!sk_item(p, chunk, h) || !sk_find(p, chunk, row0, len)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g = lane >> 4;
  const size_t group = (size_t)(h / (p.n_heads / p.n_groups)) * p.dim;
  const bf16_t* kp = p.k + (size_t)row0 * p.stride + group;
  const bf16_t* qp = p.q + (size_t)row0 * p.stride + group;
  const bf16_t* xp = p.x + (size_t)row0 * p.stride + (size_t)h * p.vdim;
  const int n_tok = (len + 31) / 32 * 32;
  for (int e = tid; e < n_tok * (NP / 8); e += 256) {
    const int j = e / (NP / 8), c = 8 * (e - j * (NP / 8));
    *reinterpret_cast<uint4*>(ks + j * KLD + c) = (j < len && c < p.dim) ? load16(kp + (size_t)j * p.stride + c) : zero16();
  }
  for (int e = tid; e < n_tok * (VP / 8); e += 256) {
    const int j = e / (VP / 8), c = 8 * (e - j * (VP / 8));
    *reinterpret_cast<uint4*>(xs + j * XLD + c) = (j < len && c < p.vdim) ? load16(xp + (size_t)j * p.stride + c) : zero16();
  }
  sk_steps(p, h, row0, len, cl, dts, &carry);          // (its barriers also stand between the tiles' writes and their reads)
  const bf16_t* sp = p.before + 2 * (((size_t)chunk * p.n_heads + h) * (NP * VP)) + 8 * lane;
  const float pass = p.d[h];
#pragma unroll
  for (int half = 0; half < 2; ++half) {
    const int i0 = 16 * (half ? 7 - wave : wave), i = i0 + c16;
    if (i0 >= len) continue;
    Frag8 qf[KN];
    const bf16_t* qrow = qp + (size_t)(i < len ? i : 0) * p.stride;
#pragma unroll
    for (int s = 0; s < KN; ++s) qf[s].u = 32 * s + 8 * g < p.dim ? load16(qrow + 32 * s + 8 * g) : zero16();
    f32x4_t acc[VT];
    const float ci = cl[i], ei = __builtin_amdgcn_exp2f(ci);
#pragma unroll
    for (int b = 0; b < VT; ++b) {
      f32x4_t a = {0.f, 0.f, 0.f, 0.f}, r = a;
#pragma unroll
      for (int s = 0; s < KN; ++s) {
        Frag8 hi, lo;
        hi.u = load16(sp + (size_t)(b * KN + s) * 1024);
        lo.u = load16(sp + (size_t)(b * KN + s) * 1024 + 512);
        a = mfma16(hi, qf[s], a);
        r = mfma16(lo, qf[s], r);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[b][e] = ei * (a[e] + r[e]);
    }
    for (int j0 = 0; j0 <= i0; j0 += 32) {
      f32x4_t s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
      for (int s = 0; s < KN; ++s) {
        Frag8 a, b;
        const uint16_t* kr = ks + (j0 + c16) * KLD + 32 * s + 8 * g;
        a.u = *reinterpret_cast<const uint4*>(kr);
        b.u = *reinterpret_cast<const uint4*>(kr + 16 * KLD);
        s0 = mfma16(a, qf[s], s0);
        s1 = mfma16(b, qf[s], s1);
      }
      float w[8];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int j = j0 + 16 * t + 4 * g;
        const float4 cj = *reinterpret_cast<const float4*>(cl + j), dj = *reinterpret_cast<const float4*>(dts + j);
        const f32x4_t& sc = t ? s1 : s0;
        w[4 * t] = j <= i ? sc[0] * dj.x * __builtin_amdgcn_exp2f(ci - cj.x) : 0.f;
        w[4 * t + 1] = j + 1 <= i ? sc[1] * dj.y * __builtin_amdgcn_exp2f(ci - cj.y) : 0.f;
        w[4 * t + 2] = j + 2 <= i ? sc[2] * dj.z * __builtin_amdgcn_exp2f(ci - cj.z) : 0.f;
        w[4 * t + 3] = j + 3 <= i ? sc[3] * dj.w * __builtin_amdgcn_exp2f(ci - cj.w) : 0.f;
      }
      Frag8 wf;
      wf.u = make_uint4(pack_bf16x2(w[0], w[1]), pack_bf16x2(w[2], w[3]), pack_bf16x2(w[4], w[5]), pack_bf16x2(w[6], w[7]));
#pragma unroll
      for (int b = 0; b < VT; ++b) acc[b] = mfma16(sk_tokens_frag(xs, XLD, j0, 16 * b), wf, acc[b]);
    }
    if (i < len) {
      float* orow = p.out + ((size_t)(row0 + i) * p.n_heads + h) * p.vdim;
#pragma unroll
      for (int b = 0; b < VT; ++b) {
        const int v = 16 * b + 4 * g;
        if (v < p.vdim) {
          const uint2 xr = *reinterpret_cast<const uint2*>(xs + i * XLD + v);
          *reinterpret_cast<float4*>(orow + v) =
              make_float4(fmaf(pass, bf16_bits_to_f32(xr.x & 0xffffu), acc[b][0]), fmaf(pass, bf16_bits_to_f32(xr.x >> 16), acc[b][1]),
                          fmaf(pass, bf16_bits_to_f32(xr.y & 0xffffu), acc[b][2]), fmaf(pass, bf16_bits_to_f32(xr.y >> 16), acc[b][3]));
        }
      }
    }
  }
}

// ---------------------------------------------------------------- entry points
static int sk_round(int v, int unit, int most) {
  int r = unit;
  while (r < v && r < most) r *= 2;
  return r;
}
extern "C" int rb_selective_chunks_ok(int dim, int vdim) {
  return dim > 0 && vdim > 0 && dim <= SK_MAX_DIM && vdim <= SK_MAX_VDIM && dim % 8 == 0 && vdim % 8 == 0;
}
extern "C" int rb_selective_chunks_most(int n_tokens, int n_seqs) { return n_tokens / SK_CHUNK + n_seqs; }
// float32 numbers of scratch: what the chunks add, the states in front of them, and their decays
extern "C" long long rb_selective_chunks_floats(int n_tokens, int n_seqs, int n_heads, int dim, int vdim) {
  const long long np = sk_round(dim, 32, SK_MAX_DIM), vp = sk_round(vdim, 32, SK_MAX_VDIM);
  const long long per = (2 * np * vp + 4) * n_heads;       // (the decays' part rounded up to 16 bytes)
  return per * rb_selective_chunks_most(n_tokens, n_seqs);
}

template <int KN, int VT>
static int sk_launch(const ScanArgs& p, hipStream_t s) {
  constexpr int NP = 32 * KN, VP = 16 * VT;
  const size_t lds1 = (size_t)SK_CHUNK * (NP + 16 + 2 * (VP + 16)) * sizeof(uint16_t);
  const size_t lds3 = (size_t)SK_CHUNK * (NP + 8 + VP + 16) * sizeof(uint16_t);
  static bool configured = false;
  if (!configured) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(scan_added_kernel<KN, VT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1);
    if (e == hipSuccess)
      e = hipFuncSetAttribute(reinterpret_cast<const void*>(scan_outputs_kernel<KN, VT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds3);
    RB_REQUIRE(e == hipSuccess, "rb_selective_chunks: cannot reserve %zu bytes of LDS: %s", lds1, hipGetErrorString(e));
    configured = true;
  }
  const int per = (p.n_chunks * p.n_heads + 7) / 8;
  scan_added_kernel<KN, VT><<<8 * per, 256, lds1, s>>>(p);
  scan_carry_kernel<KN, VT><<<dim3(p.n_seqs, p.n_heads, (NP * VP / 8 + 255) / 256), 256, 0, s>>>(p);
  scan_outputs_kernel<KN, VT><<<8 * per, 256, lds3, s>>>(p);
  return 0;
}

extern "C" int rb_selective_chunks(const void* q, const void* k, const void* x, long long stride, const float* dt_in, long long dt_stride,
                                   const float* dt_bias, const float* a_log, const float* d, float* state, const int32_t* cu_seqlens,
                                   const int32_t* slots, float* scratch, float* out, int n_seqs, int n_tokens, int n_heads, int n_groups,
                                   int dim, int vdim, void* stream) {
  RB_RECORDED(rb_selective_chunks(q, k, x, stride, dt_in, dt_stride, dt_bias, a_log, d, state, cu_seqlens, slots, scratch, out, n_seqs,
                                  n_tokens, n_heads, n_groups, dim, vdim, stream));
  RB_REQUIRE(n_seqs >= 0 && n_tokens >= 0 && n_heads > 0 && n_heads <= 65535 && n_groups > 0 && n_heads % n_groups == 0,
             "rb_selective_chunks: bad sizes B=%d T=%d H=%d groups=%d", n_seqs, n_tokens, n_heads, n_groups);
  RB_REQUIRE(rb_selective_chunks_ok(dim, vdim),
             "rb_selective_chunks: a state of %d x %d not supported (multiples of 8 up to %d and %d; use rb_selective_scan)", dim, vdim,
             SK_MAX_DIM, SK_MAX_VDIM);
  RB_REQUIRE(stride >= (long long)n_heads * vdim && stride >= (long long)n_groups * dim && stride % 8 == 0 && dt_stride >= n_heads,
             "rb_selective_chunks: a row stride is too short, or no multiple of 8");
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  RB_REQUIRE(aligned(q) && aligned(k) && aligned(x) && aligned(out) && aligned(state) && aligned(scratch),
             "rb_selective_chunks: operands must be 16-byte aligned");
  const long long n_chunks = rb_selective_chunks_most(n_tokens, n_seqs);
  RB_REQUIRE((n_chunks * n_heads + 7) / 8 * 8 <= 0x7fffffffLL, "rb_selective_chunks: too many chunks");
  if (n_seqs == 0 || n_tokens == 0) return 0;
  const int np = sk_round(dim, 32, SK_MAX_DIM), vp = sk_round(vdim, 32, SK_MAX_VDIM);
  const size_t per = (size_t)n_chunks * n_heads;
  float* added = scratch;
  bf16_t* before = reinterpret_cast<bf16_t*>(scratch + per * np * vp);
  float* total = scratch + 2 * per * np * vp;
  const ScanArgs p = {(const bf16_t*)x, (const bf16_t*)k, (const bf16_t*)q, (size_t)stride, dt_in, (size_t)dt_stride, dt_bias, a_log, d, state,
                      cu_seqlens, slots, out, added, before, total, n_seqs, n_heads, n_groups, dim, vdim, (int)n_chunks};
  hipStream_t s = (hipStream_t)stream;
  int rc = 1;
#define SK_BY_V(KN) (vp == 32 ? sk_launch<KN, 2>(p, s) : vp == 64 ? sk_launch<KN, 4>(p, s) : sk_launch<KN, 8>(p, s))
  if (np == 32) rc = SK_BY_V(1);
  else if (np == 64) rc = SK_BY_V(2);
  else if (np == 128) rc = SK_BY_V(4);
  else rc = SK_BY_V(8);
#undef SK_BY_V
  if (rc) return rc;
  RB_LAUNCH_CHECK();
  return 0;
}
