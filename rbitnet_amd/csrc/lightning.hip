// Linear attention with one constant decay per head, for steps that bring several tokens of a sequence:
//   S_t = d S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t,   q, k, v behind silu, d the head's decay,
// with the tokens of a piece taken in chunks of 64 on the matrix cores, in float32 (16x16x4: float32 inputs, products and
// sums).  For token i of a chunk of L tokens (i = 0 .. L - 1), with S the state before the chunk:
//   o_i = sum_(j <= i) d^(i - j) (q_i . k_j) v_j  +  S^T (d^(i + 1) q_i)          S' = d^L S + sum_j (d^(L - 1 - j) k_j) v_j^T
// Two launches.  The first takes every chunk and head by itself: silu, the sum inside the chunk, and what the second needs,
// d^(i + 1) q_i, d^(L - 1 - j) k_j and v_j, written over the projections they came from.  The second walks a sequence's chunks
// one after the other with 16 columns of a head's state a workgroup: the read-out of the state before the chunk, added to what
// the first left, and the state's update; a chunk there is two products of 64 tokens and one barrier.
// A chunk is counted from the start of a sequence's piece of the step; the results do not depend on how the tokens were
// cut beyond rounding.  powers [H][65] holds d^0 .. d^64.
#include <math.h>

#include "api.h"
#include "common.h"
#include "mfma.h"

#define LN_CHUNK 64
#define LN_POWERS (LN_CHUNK + 1)
#define LN_MAX_DIM 128

__device__ __forceinline__ f32x4_t mfma16_f32(float a, float b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ float ln_silu(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float4 ln_silu4(const float4& v) { return make_float4(ln_silu(v.x), ln_silu(v.y), ln_silu(v.z), ln_silu(v.w)); }
__device__ __forceinline__ float4 ln_scale4(const float4& v, float f) { return make_float4(v.x * f, v.y * f, v.z * f, v.w * f); }

// The sequence and the first token (within the step's rows) of chunk `at` of the step: sequences one after the other, each
// with as many chunks as its piece fills.  false: past the end.
__device__ __forceinline__ bool ln_find(const int32_t* __restrict__ cu, int n_seqs, int at, int& row0, int& len) {
  for (int b = 0; b < n_seqs; ++b) {
    const int n = cu[b + 1] - cu[b], chunks = (n + LN_CHUNK - 1) / LN_CHUNK;
    if (at < chunks) {
      row0 = cu[b] + at * LN_CHUNK;
      len = n - at * LN_CHUNK < LN_CHUNK ? n - at * LN_CHUNK : LN_CHUNK;
      return true;
    }
    at -= chunks;
  }
  return false;
}

// ---------------------------------------------------------------- inside a chunk
// DK, DV: dim and vdim rounded up to 64 or 128 (zeros beyond).  A workgroup of 4 waves takes a chunk and a head; k and v of
// the chunk lie in LDS; wave w takes queries 16 w .. 16 w + 15: scores transposed (keys x queries), so that they come out of
// the first product in the layout that the second wants.  A product's depth is counted so that lane group g of step 16 s + j
// takes 16 s + 4 g + j: four steps' operands are then 16 bytes in a row.
template <int DK, int DV>
__global__ __launch_bounds__(256) void lightning_inner_kernel(float* __restrict__ q, float* __restrict__ k, size_t qk_stride,
                                                              float* __restrict__ v, size_t v_stride, const float* __restrict__ powers,
                                                              const int32_t* __restrict__ cu_seqlens, int n_seqs,
                                                              float* __restrict__ out, int n_heads, int dim, int vdim) {
  constexpr int KLD = DK + 4, VLD = DV + 4;      // rows 4 banks on from a multiple of 64: neither read below hits a bank twice
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* ks = lds;                               // [64][KLD]
  float* vs = lds + LN_CHUNK * KLD;              // [64][VLD]
  __shared__ float pw[LN_POWERS];
  int row0, len;
  if (!ln_find(cu_seqlens, n_seqs, blockIdx.x, row0, len)) return;
  const int h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c16 = lane & 15, g = lane >> 4;
  if (tid < LN_POWERS) pw[tid] = powers[(size_t)h * LN_POWERS + tid];
  __syncthreads();
  // ---- this wave's queries, k and v of the chunk: through silu, and written back as the second launch reads them
  const int qi = 16 * wave + c16;                // this lane's query
  const bool q_on = qi < len;
  float4 qf[DK / 16];
  {
    float* qrow = q + (size_t)(row0 + (q_on ? qi : 0)) * qk_stride + (size_t)h * dim;
#pragma unroll
    for (int s = 0; s < DK / 16; ++s) {
      const int d = 16 * s + 4 * g;
      qf[s] = (q_on && d < dim) ? *reinterpret_cast<const float4*>(qrow + d) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int s = 0; s < DK / 16; ++s) {
      const int d = 16 * s + 4 * g;
      qf[s] = ln_silu4(qf[s]);
      if (q_on && d < dim) *reinterpret_cast<float4*>(qrow + d) = ln_scale4(qf[s], pw[qi + 1]);
    }
  }
  for (int e = tid; e < LN_CHUNK * (DK / 4); e += 256) {
    const int j = e / (DK / 4), d = 4 * (e - j * (DK / 4));
    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
    if (j < len && d < dim) {
      float* p = k + (size_t)(row0 + j) * qk_stride + (size_t)h * dim + d;
      x = ln_silu4(*reinterpret_cast<const float4*>(p));
      *reinterpret_cast<float4*>(p) = ln_scale4(x, pw[len - 1 - j]);
    }
    *reinterpret_cast<float4*>(ks + j * KLD + d) = x;
  }
  for (int e = tid; e < LN_CHUNK * (DV / 4); e += 256) {
    const int j = e / (DV / 4), d = 4 * (e - j * (DV / 4));
    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
    if (j < len && d < vdim) {
      float* p = v + (size_t)(row0 + j) * v_stride + (size_t)h * vdim + d;
      x = ln_silu4(*reinterpret_cast<const float4*>(p));
      *reinterpret_cast<float4*>(p) = x;
    }
    *reinterpret_cast<float4*>(vs + j * VLD + d) = x;
  }
  __syncthreads();
  if (16 * wave >= len) return;
  f32x4_t acc[DV / 16];
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt) acc[dt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int kt = 0; kt <= wave; ++kt) {           // tiles of 16 keys up to the diagonal's
    f32x4_t sc = {0.f, 0.f, 0.f, 0.f}, sc2 = sc;
#pragma unroll
    for (int s = 0; s < DK / 16; ++s) {
      const float4 kf = *reinterpret_cast<const float4*>(ks + (16 * kt + c16) * KLD + 16 * s + 4 * g);
      sc = mfma16_f32(kf.x, qf[s].x, sc);
      sc2 = mfma16_f32(kf.y, qf[s].y, sc2);
      sc = mfma16_f32(kf.z, qf[s].z, sc);
      sc2 = mfma16_f32(kf.w, qf[s].w, sc2);
    }
    float p[4];                                  // keys 16 kt + 4 g + i of query qi
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int back = qi - (16 * kt + 4 * g + i);
      p[i] = back >= 0 ? (sc[i] + sc2[i]) * pw[back] : 0.f;
    }
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[dt] = mfma16_f32(vs[(16 * kt + 4 * g + i) * VLD + 16 * dt + c16], p[i], acc[dt]);
  }
  if (!q_on) return;
  float* orow = out + ((size_t)(row0 + qi) * n_heads + h) * vdim;
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt) {
    const int d = 16 * dt + 4 * g;
    if (d < vdim) *reinterpret_cast<float4*>(orow + d) = make_float4(acc[dt][0], acc[dt][1], acc[dt][2], acc[dt][3]);
  }
}

// ---------------------------------------------------------------- from chunk to chunk
// A workgroup of 4 waves holds 16 columns (value channels) of a head's state: wave w rows 16 RT w .. of it in its
// accumulators (RT tiles of 16 rows; with two, row r of tile i is number 32 w + 2 r + i of the head, so that a lane's operand
// of both tiles is 8 bytes in a row), and all of them in LDS, twice, for every wave's read-out.  A chunk's operands are asked
// for two chunks ahead.
template <int DK>
__global__ __launch_bounds__(256) void lightning_carry_kernel(const float* __restrict__ q, const float* __restrict__ k, size_t qk_stride,
                                                              const float* __restrict__ v, size_t v_stride,
                                                              const float* __restrict__ powers, float* __restrict__ state,
                                                              const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots,
                                                              float* __restrict__ out, int n_heads, int dim, int vdim) {
  constexpr int RT = DK / 64, SLD = DK + 4;
  __shared__ __attribute__((aligned(16))) float st[2][16 * SLD];      // [column][row]
  const int b = blockIdx.x, h = blockIdx.y, col0 = 16 * blockIdx.z;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c16 = lane & 15, g = lane >> 4;
  const int seq0 = cu_seqlens[b], n = cu_seqlens[b + 1] - seq0;
  if (n <= 0) return;
  const int col = col0 + c16;
  const bool col_on = col < vdim;
  float* S = state + (((size_t)slots[b] * n_heads + h) * vdim + (col_on ? col : 0)) * dim;
  // this lane's rows of column `col`: 4 RT of them in a row
  const int r_lane = 16 * RT * wave + 4 * RT * g;
  f32x4_t acc[RT];
  {
    float own[4 * RT];
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int r = r_lane + 4 * i;
      const float4 x = (col_on && r < dim) ? *reinterpret_cast<const float4*>(S + r) : make_float4(0.f, 0.f, 0.f, 0.f);
      own[4 * i] = x.x;
      own[4 * i + 1] = x.y;
      own[4 * i + 2] = x.z;
      own[4 * i + 3] = x.w;
      *reinterpret_cast<float4*>(&st[0][c16 * SLD + r]) = x;
    }
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[i][e] = own[RT * e + i];
  }
  // Loads are unconditional, from an address inside the step where a token, row or column lies outside, so that they are all in
  // flight together: a query or column that is not there gives a result that nobody stores; a token that is not there must not
  // reach the state (its v becomes 0 at use), nor a row of the head beyond dim the read-out (its q becomes 0 at use).
  struct Chunk {
    float4 q[DK / 16];        // query 16 w + c16: rows 16 s + 4 g ..
    float k[16][RT];          // token 4 s + g: rows of this wave's tiles
    float v[16];              // token 4 s + g: this lane's column
    float o[4];               // queries 16 w + 4 g + i: what the first launch left
  };
  const int k_row = 16 * RT * wave + RT * c16;
  const float* q_base = q + (size_t)h * dim;
  const float* k_base = k + (size_t)h * dim + (k_row < dim ? k_row : 0);
  const float* v_base = v + (size_t)h * vdim + (col_on ? col : 0);
  const size_t o_base = (size_t)h * vdim + (col_on ? col : 0), o_stride = (size_t)n_heads * vdim;
  auto fetch = [&](Chunk& x, int at) {
    const int len = n - at < LN_CHUNK ? n - at : LN_CHUNK;
    const size_t row0 = (size_t)(seq0 + at);
    const int qi = 16 * wave + c16;
    const float* qrow = q_base + (row0 + (qi < len ? qi : 0)) * qk_stride;
#pragma unroll
    for (int s = 0; s < DK / 16; ++s) {
      const int d = 16 * s + 4 * g;
      x.q[s] = *reinterpret_cast<const float4*>(qrow + (d < dim ? d : 0));
    }
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      const size_t t = row0 + (4 * s + g < len ? 4 * s + g : 0);
      if (RT == 2) {
        const float2 two = *reinterpret_cast<const float2*>(k_base + t * qk_stride);
        x.k[s][0] = two.x;
        x.k[s][RT - 1] = two.y;
      } else {
        x.k[s][0] = k_base[t * qk_stride];
      }
      x.v[s] = v_base[t * v_stride];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      x.o[i] = out[(row0 + (t < len ? t : 0)) * o_stride + o_base];
    }
    __builtin_amdgcn_sched_barrier(0);            // asked for here, not where the scheduler would sink them: at their use
  };
  int buf = 0;
  // chunk at token `at` from `cur`, while the chunk two further on is fetched into `later`
  auto work = [&](Chunk& cur, Chunk& later, int at) {
    const int len = n - at < LN_CHUNK ? n - at : LN_CHUNK;
    const bool more = at + LN_CHUNK < n;
    __syncthreads();                              // the state of all waves' rows is there
    if (at + 2 * LN_CHUNK < n) fetch(later, at + 2 * LN_CHUNK);
    const float dl = powers[(size_t)h * LN_POWERS + len];
    if (dim < DK) {
#pragma unroll
      for (int s = 0; s < DK / 16; ++s)
        if (16 * s + 4 * g >= dim) cur.q[s] = make_float4(0.f, 0.f, 0.f, 0.f);
    }
    if (len < LN_CHUNK) {
#pragma unroll
      for (int s = 0; s < 16; ++s)
        if (4 * s + g >= len) cur.v[s] = 0.f;
    }
    f32x4_t oa = {cur.o[0], cur.o[1], cur.o[2], cur.o[3]}, ob = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[i][e] *= dl;
#pragma unroll
    for (int s = 0; s < 16; ++s)
#pragma unroll
      for (int i = 0; i < RT; ++i) acc[i] = mfma16_f32(cur.k[s][i], cur.v[s], acc[i]);
#pragma unroll
    for (int s = 0; s < DK / 16; ++s) {
      const float4 sf = *reinterpret_cast<const float4*>(&st[buf][c16 * SLD + 16 * s + 4 * g]);
      oa = mfma16_f32(cur.q[s].x, sf.x, oa);
      ob = mfma16_f32(cur.q[s].y, sf.y, ob);
      oa = mfma16_f32(cur.q[s].z, sf.z, oa);
      ob = mfma16_f32(cur.q[s].w, sf.w, ob);
    }
    if (more) {
      float own[4 * RT];
#pragma unroll
      for (int i = 0; i < RT; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) own[RT * e + i] = acc[i][e];
#pragma unroll
      for (int i = 0; i < RT; ++i)
        *reinterpret_cast<float4*>(&st[buf ^ 1][c16 * SLD + r_lane + 4 * i]) = make_float4(own[4 * i], own[4 * i + 1], own[4 * i + 2], own[4 * i + 3]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      if (t < len && col_on) out[(size_t)(seq0 + at + t) * o_stride + o_base] = oa[i] + ob[i];
    }
    buf ^= 1;
  };
  // three chunks' operands in registers: the one at work and two on their way
  Chunk x0, x1, x2;
  fetch(x0, 0);
  if (LN_CHUNK < n) fetch(x1, LN_CHUNK);
  for (int at = 0; at < n; at += 3 * LN_CHUNK) {
    work(x0, x2, at);
    if (at + LN_CHUNK < n) work(x1, x0, at + LN_CHUNK);
    if (at + 2 * LN_CHUNK < n) work(x2, x1, at + 2 * LN_CHUNK);
  }
  if (!col_on) return;
  float own[4 * RT];
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) own[RT * e + i] = acc[i][e];
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int r = r_lane + 4 * i;
    if (r < dim) *reinterpret_cast<float4*>(S + r) = make_float4(own[4 * i], own[4 * i + 1], own[4 * i + 2], own[4 * i + 3]);
  }
}

extern "C" int rb_lightning_chunks_ok(int dim, int vdim) {
  return dim > 0 && vdim > 0 && dim <= LN_MAX_DIM && vdim <= LN_MAX_DIM && dim % 4 == 0 && vdim % 4 == 0;
}

template <int DK, int DV>
static int launch_inner(float* q, float* k, size_t qs, float* v, size_t vs, const float* powers, const int32_t* cu, int n_seqs, float* out,
                        int n_tokens, int n_heads, int dim, int vdim, hipStream_t s) {
  const size_t lds = (size_t)LN_CHUNK * (DK + 4 + DV + 4) * sizeof(float);
  auto kern = lightning_inner_kernel<DK, DV>;
  static bool configured = false;
  if (!configured) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    RB_REQUIRE(e == hipSuccess, "rb_lightning_chunks: cannot reserve %zu bytes of LDS: %s", lds, hipGetErrorString(e));
    configured = true;
  }
  kern<<<dim3(n_tokens / LN_CHUNK + n_seqs, n_heads), 256, lds, s>>>(q, k, qs, v, vs, powers, cu, n_seqs, out, n_heads, dim, vdim);
  return 0;
}

// q, k [T, H dim] and v [T, H vdim] float32 (rows qk_stride and v_stride apart) are overwritten.
extern "C" int rb_lightning_chunks(float* q, float* k, long long qk_stride, float* v, long long v_stride, const float* powers, float* state,
                                   const int32_t* cu_seqlens, const int32_t* slots, float* out, int n_seqs, int n_tokens, int n_heads,
                                   int dim, int vdim, void* stream) {
  RB_RECORDED(rb_lightning_chunks(q, k, qk_stride, v, v_stride, powers, state, cu_seqlens, slots, out, n_seqs, n_tokens, n_heads, dim, vdim,
                                  stream));
  RB_REQUIRE(n_seqs >= 0 && n_tokens >= 0 && n_heads > 0 && n_heads <= 65535, "rb_lightning_chunks: bad sizes B=%d T=%d H=%d", n_seqs,
             n_tokens, n_heads);
  RB_REQUIRE(rb_lightning_chunks_ok(dim, vdim), "rb_lightning_chunks: heads of %d and %d numbers not supported (multiples of 4 up to %d; use rb_lightning_recurrence)",
             dim, vdim, LN_MAX_DIM);
  RB_REQUIRE(qk_stride >= (long long)n_heads * dim && v_stride >= (long long)n_heads * vdim, "rb_lightning_chunks: a row stride is too short");
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  RB_REQUIRE(aligned(q) && aligned(k) && aligned(v) && aligned(out) && aligned(state) && qk_stride % 4 == 0 && v_stride % 4 == 0,
             "rb_lightning_chunks: rows must be 16-byte aligned");
  if (n_seqs == 0 || n_tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const size_t qs = (size_t)qk_stride, vs = (size_t)v_stride;
  int rc;
  if (dim <= 64)
    rc = vdim <= 64 ? launch_inner<64, 64>(q, k, qs, v, vs, powers, cu_seqlens, n_seqs, out, n_tokens, n_heads, dim, vdim, s)
                    : launch_inner<64, 128>(q, k, qs, v, vs, powers, cu_seqlens, n_seqs, out, n_tokens, n_heads, dim, vdim, s);
  else
    rc = vdim <= 64 ? launch_inner<128, 64>(q, k, qs, v, vs, powers, cu_seqlens, n_seqs, out, n_tokens, n_heads, dim, vdim, s)
                    : launch_inner<128, 128>(q, k, qs, v, vs, powers, cu_seqlens, n_seqs, out, n_tokens, n_heads, dim, vdim, s);
  if (rc) return rc;
  dim3 grid(n_seqs, n_heads, (vdim + 15) / 16);
  if (dim <= 64)
    lightning_carry_kernel<64><<<grid, 256, 0, s>>>(q, k, qs, v, vs, powers, state, cu_seqlens, slots, out, n_heads, dim, vdim);
  else
    lightning_carry_kernel<128><<<grid, 256, 0, s>>>(q, k, qs, v, vs, powers, state, cu_seqlens, slots, out, n_heads, dim, vdim);
  RB_LAUNCH_CHECK();
  return 0;
}
