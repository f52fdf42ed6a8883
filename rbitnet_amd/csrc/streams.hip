// A residual stream kept as several copies (hyper-connections), layer norm with weight and bias, and two small
// element-wise functions: the xIELU activation and the tanh cap of logits.  float32 arithmetic throughout.
//
// (The kernels for RMS norms of such streams take an update's term as a sum of terms as well.)
// The streams are x [S, T, E], stream_stride floats from one copy to the next.  A sublayer reads the mixture
// u = sum_s coef[s] x[s], and afterwards every copy is rebuilt from all the old ones:
//   x'[j] = sum_s mix[s, j] x[s] + out[j] * (scale * y)
// One stream with coef = mix = out = 1 is the plain residual sum.
#include <math.h>

#include "api.h"
#include "common.h"

#define ST_MAX_STREAMS 16

// out[r] = (u - mean(u)) / sqrt(mean((u - mean)^2) + eps) * weight + bias, u = sum_s coef[s] x[s][src] (+ delta[src]),
// src = rows ? rows[r] : r.  With one stream, a delta and no rows the sum is written back to x (the residual sum of
// a plain pre-norm layer).  coef null: every coefficient is 1.  bias null: none.  The row is held in LDS between
// the passes: mean first, then the squared deviations.
template <typename TO>
__global__ void streams_layernorm_kernel(float* __restrict__ x, int n_streams, size_t stream_stride,
                                         const float* __restrict__ coef, const float* __restrict__ delta,
                                         const float* __restrict__ weight, const float* __restrict__ bias, float eps,
                                         const int32_t* __restrict__ rows, int width, TO* __restrict__ out,
                                         const float* __restrict__ mix, const float* __restrict__ out_coef,
                                         const float* __restrict__ y, const float* __restrict__ scale,
                                         const float* __restrict__ delta2, float dscale) {
  extern __shared__ float u[];
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : (size_t)r;
  const bool write_back = delta != nullptr && rows == nullptr && n_streams == 1;
  float sum = 0.f;
  for (int j = threadIdx.x; j < width; j += blockDim.x) {
    float v = 0.f;
    if (mix) {
      // the update that was still to be done: every copy from all the old ones, then the mixture of the new ones
      float old[ST_MAX_STREAMS];
#pragma unroll
      for (int s = 0; s < ST_MAX_STREAMS; ++s)
        if (s < n_streams) old[s] = x[(size_t)s * stream_stride + src * width + j];
      float yv = y[src * width + j];
      if (scale) yv *= scale[j];
#pragma unroll
      for (int k = 0; k < ST_MAX_STREAMS; ++k) {
        if (k < n_streams) {
          float nv = out_coef[k] * yv;
#pragma unroll
          for (int s = 0; s < ST_MAX_STREAMS; ++s)
            if (s < n_streams) nv = fmaf(mix[s * n_streams + k], old[s], nv);
          x[(size_t)k * stream_stride + src * width + j] = nv;
          v = coef ? fmaf(coef[k], nv, v) : v + nv;
        }
      }
    } else {
      for (int s = 0; s < n_streams; ++s) {
        const float xv = x[(size_t)s * stream_stride + src * width + j];
        v = coef ? fmaf(coef[s], xv, v) : v + xv;
      }
    }
    if (delta) v = fmaf(dscale, delta2 ? delta[src * width + j] + delta2[src * width + j] : delta[src * width + j], v);
    if (write_back) x[src * width + j] = v;
    u[j] = v;
    sum += v;
  }
  const float mean = block_sum(sum, scratch) / (float)width;
  float ss = 0.f;
  for (int j = threadIdx.x; j < width; j += blockDim.x) {
    const float d = u[j] - mean;
    ss = fmaf(d, d, ss);
  }
  const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
  TO* orow = out + (size_t)r * width;
  for (int j = threadIdx.x; j < width; j += blockDim.x) {
    const float v = (u[j] - mean) * f * weight[j];
    Num<TO>::store(orow + j, bias ? v + bias[j] : v);
  }
}

// The same for widths that are multiples of 4, four values a thread with 16-byte loads and up to 1024 threads a row,
// so that a row's loads are all in flight together (a step of few tokens has few rows, and their time is the
// chain of trips to memory).
__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 fma4(float a, const float4& b, const float4& c) {
  return make_float4(fmaf(a, b.x, c.x), fmaf(a, b.y, c.y), fmaf(a, b.z, c.z), fmaf(a, b.w, c.w));
}
__device__ __forceinline__ void st4(float* p, float a, float b, float c, float d) { *reinterpret_cast<float4*>(p) = make_float4(a, b, c, d); }
__device__ __forceinline__ void st4(bf16_t* p, float a, float b, float c, float d) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
}

template <typename TO>
__global__ __launch_bounds__(1024) void streams_layernorm_vec_kernel(
    float* __restrict__ x, int n_streams, size_t stream_stride, const float* __restrict__ coef, const float* __restrict__ delta,
    const float* __restrict__ weight, const float* __restrict__ bias, float eps, const int32_t* __restrict__ rows, int width,
    TO* __restrict__ out, const float* __restrict__ mix, const float* __restrict__ out_coef, const float* __restrict__ y,
    const float* __restrict__ scale, const float* __restrict__ delta2, float dscale) {
  extern __shared__ float u[];
  __shared__ float scratch[16];
  __shared__ float c_mix[ST_MAX_STREAMS * ST_MAX_STREAMS], c_out[ST_MAX_STREAMS], c_in[ST_MAX_STREAMS];
  const int r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : (size_t)r;
  const bool write_back = delta != nullptr && rows == nullptr && n_streams == 1;
  if ((int)threadIdx.x < n_streams) {
    c_in[threadIdx.x] = coef ? coef[threadIdx.x] : 1.0f;
    if (mix) c_out[threadIdx.x] = out_coef[threadIdx.x];
  }
  if (mix && (int)threadIdx.x < n_streams * n_streams) c_mix[threadIdx.x] = mix[threadIdx.x];
  __syncthreads();
  float sum = 0.f;
  for (int j = 4 * threadIdx.x; j < width; j += 4 * blockDim.x) {
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (mix) {
      float4 old[ST_MAX_STREAMS];
#pragma unroll
      for (int s = 0; s < ST_MAX_STREAMS; ++s)
        if (s < n_streams) old[s] = ld4(x + (size_t)s * stream_stride + src * width + j);
      float4 yv = ld4(y + src * width + j);
      if (scale) {
        const float4 sc = ld4(scale + j);
        yv = make_float4(yv.x * sc.x, yv.y * sc.y, yv.z * sc.z, yv.w * sc.w);
      }
#pragma unroll
      for (int k = 0; k < ST_MAX_STREAMS; ++k) {
        if (k < n_streams) {
          const float oc = c_out[k];
          float4 nv = make_float4(oc * yv.x, oc * yv.y, oc * yv.z, oc * yv.w);
#pragma unroll
          for (int s = 0; s < ST_MAX_STREAMS; ++s)
            if (s < n_streams) nv = fma4(c_mix[s * n_streams + k], old[s], nv);
          *reinterpret_cast<float4*>(x + (size_t)k * stream_stride + src * width + j) = nv;
          v = fma4(c_in[k], nv, v);
        }
      }
    } else {
#pragma unroll
      for (int s = 0; s < ST_MAX_STREAMS; ++s)
        if (s < n_streams) v = fma4(c_in[s], ld4(x + (size_t)s * stream_stride + src * width + j), v);
    }
    if (delta) {
      float4 d = ld4(delta + src * width + j);
      if (delta2) {
        const float4 e = ld4(delta2 + src * width + j);
        d = make_float4(d.x + e.x, d.y + e.y, d.z + e.z, d.w + e.w);
      }
      v = fma4(dscale, d, v);
    }
    if (write_back) *reinterpret_cast<float4*>(x + src * width + j) = v;
    *reinterpret_cast<float4*>(u + j) = v;
    sum += (v.x + v.y) + (v.z + v.w);
  }
  // weight and bias of this thread's first values are asked for now, so that they arrive under the two reductions
  const int j0 = 4 * threadIdx.x;
  float4 w0 = make_float4(0.f, 0.f, 0.f, 0.f), b0 = w0;
  if (j0 < width) {
    w0 = ld4(weight + j0);
    if (bias) b0 = ld4(bias + j0);
  }
  __builtin_amdgcn_sched_barrier(0);
  const float mean = block_sum(sum, scratch) / (float)width;
  float ss = 0.f;
  for (int j = 4 * threadIdx.x; j < width; j += 4 * blockDim.x) {
    const float4 v = *reinterpret_cast<const float4*>(u + j);
    const float a = v.x - mean, b = v.y - mean, c = v.z - mean, d = v.w - mean;
    ss += (a * a + b * b) + (c * c + d * d);
  }
  const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
  TO* orow = out + (size_t)r * width;
  for (int j = 4 * threadIdx.x; j < width; j += 4 * blockDim.x) {
    const float4 v = *reinterpret_cast<const float4*>(u + j);
    const float4 wv = j == j0 ? w0 : ld4(weight + j);
    float4 o = make_float4((v.x - mean) * f * wv.x, (v.y - mean) * f * wv.y, (v.z - mean) * f * wv.z, (v.w - mean) * f * wv.w);
    if (bias) {
      const float4 bv = j == j0 ? b0 : ld4(bias + j);
      o = make_float4(o.x + bv.x, o.y + bv.y, o.z + bv.z, o.w + bv.w);
    }
    st4(orow + j, o.x, o.y, o.z, o.w);
  }
}

extern "C" int rb_streams_layernorm(float* x, int n_streams, long long stream_stride, const float* coef,
                                    const float* delta, const float* weight, const float* bias, float eps,
                                    const int32_t* rows, int n_rows, int width, void* out, int out_dtype, void* stream) {
  return rb_streams_update_layernorm(x, n_streams, stream_stride, nullptr, nullptr, nullptr, nullptr, coef, delta, weight, bias,
                                     eps, rows, n_rows, width, out, out_dtype, stream);
}

// The same after an update of the copies that was still to be done (rb_streams_update's mix, out_coef, y, scale; mix
// null: none), in one pass over the rows: the copies are rewritten and the norm reads the new ones.  With an update
// every row is taken (rows must be null).
static int layernorm_launch(float* x, int n_streams, long long stream_stride, const float* mix, const float* out_coef, const float* y,
                            const float* scale, const float* coef, const float* delta, const float* delta2, float dscale,
                            const float* weight, const float* bias, float eps, const int32_t* rows, int n_rows, int width, void* out,
                            int out_dtype, void* stream);

extern "C" int rb_streams_update_layernorm(float* x, int n_streams, long long stream_stride, const float* mix,
                                           const float* out_coef, const float* y, const float* scale, const float* coef,
                                           const float* delta, const float* weight, const float* bias, float eps,
                                           const int32_t* rows, int n_rows, int width, void* out, int out_dtype,
                                           void* stream) {
  RB_RECORDED(rb_streams_update_layernorm(x, n_streams, stream_stride, mix, out_coef, y, scale, coef, delta, weight, bias, eps,
                                          rows, n_rows, width, out, out_dtype, stream));
  return layernorm_launch(x, n_streams, stream_stride, mix, out_coef, y, scale, coef, delta, nullptr, 1.0f, weight, bias, eps, rows,
                          n_rows, width, out, out_dtype, stream);
}

// Layer norm of a plain stream x [T, E] with the residual sum that was still to be done, in one pass:
//   v = x[src] + dscale * (delta[src] + (delta2 ? delta2[src] : 0)),  src = rows ? rows[r] : r;  without rows x[src] = v as well;
//   out[r] = (v - mean) / sqrt(var + eps) * weight + bias.   delta null: the norm alone.
extern "C" int rb_layernorm_residual(float* x, const float* delta, const float* delta2, float dscale, const float* weight,
                                     const float* bias, float eps, const int32_t* rows, int n_rows, int width, void* out,
                                     int out_dtype, void* stream) {
  RB_RECORDED(rb_layernorm_residual(x, delta, delta2, dscale, weight, bias, eps, rows, n_rows, width, out, out_dtype, stream));
  RB_REQUIRE(delta != nullptr || delta2 == nullptr, "rb_layernorm_residual: a second term without a first");
  return layernorm_launch(x, 1, 0, nullptr, nullptr, nullptr, nullptr, nullptr, delta, delta2, dscale, weight, bias, eps, rows, n_rows,
                          width, out, out_dtype, stream);
}

static int layernorm_launch(float* x, int n_streams, long long stream_stride, const float* mix, const float* out_coef, const float* y,
                            const float* scale, const float* coef, const float* delta, const float* delta2, float dscale,
                            const float* weight, const float* bias, float eps, const int32_t* rows, int n_rows, int width, void* out,
                            int out_dtype, void* stream) {
  RB_REQUIRE(mix == nullptr || (rows == nullptr && out_coef != nullptr && y != nullptr),
             "rb_streams_update_layernorm: an update takes every row and needs out_coef and y");
  RB_REQUIRE(n_rows >= 0 && width > 0 && width <= 16384, "rb_streams_layernorm: bad sizes %d x %d (width at most 16384)", n_rows, width);
  RB_REQUIRE(n_streams >= 1 && n_streams <= ST_MAX_STREAMS && stream_stride >= 0, "rb_streams_layernorm: %d streams (1 to %d)",
             n_streams, ST_MAX_STREAMS);
  if (n_rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const size_t lds = (size_t)width * sizeof(float);
  auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (width % 4 == 0 && stream_stride % 4 == 0 && aligned(x) && aligned(delta) && aligned(delta2) && aligned(weight) && aligned(bias) && aligned(out) &&
      aligned(y) && aligned(scale) && (out_dtype == RB_F32 || out_dtype == RB_BF16)) {
    int threads = ((width / 4 + RB_WAVE - 1) / RB_WAVE) * RB_WAVE;
    if (threads > 1024) threads = 1024;
    if (out_dtype == RB_F32)
      streams_layernorm_vec_kernel<float><<<n_rows, threads, lds, s>>>(x, n_streams, (size_t)stream_stride, coef, delta, weight, bias,
                                                                       eps, rows, width, (float*)out, mix, out_coef, y, scale, delta2, dscale);
    else
      streams_layernorm_vec_kernel<bf16_t><<<n_rows, threads, lds, s>>>(x, n_streams, (size_t)stream_stride, coef, delta, weight,
                                                                        bias, eps, rows, width, (bf16_t*)out, mix, out_coef, y, scale, delta2, dscale);
    RB_LAUNCH_CHECK();
    return 0;
  }
  if (out_dtype == RB_F32)
    streams_layernorm_kernel<float><<<n_rows, 256, lds, s>>>(x, n_streams, (size_t)stream_stride, coef, delta, weight, bias, eps,
                                                             rows, width, (float*)out, mix, out_coef, y, scale, delta2, dscale);
  else if (out_dtype == RB_BF16)
    streams_layernorm_kernel<bf16_t><<<n_rows, 256, lds, s>>>(x, n_streams, (size_t)stream_stride, coef, delta, weight, bias, eps,
                                                              rows, width, (bf16_t*)out, mix, out_coef, y, scale, delta2, dscale);
  else
    RB_REQUIRE(false, "rb_streams_layernorm: unknown dtype %d", out_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}

// x'[j] = sum_s mix[s, j] x[s] + out_coef[j] * scale * y for all copies j at once; a thread owns an element of
// all copies, reads them, then writes them.
__global__ void streams_update_kernel(float* __restrict__ x, int n_streams, size_t stream_stride,
                                      const float* __restrict__ mix, const float* __restrict__ out_coef,
                                      const float* __restrict__ y, const float* __restrict__ scale, int width,
                                      size_t n_elems) {
  for (size_t e = (size_t)blockIdx.x * blockDim.x + threadIdx.x; e < n_elems; e += (size_t)gridDim.x * blockDim.x) {
    float old[ST_MAX_STREAMS];
#pragma unroll
    for (int s = 0; s < ST_MAX_STREAMS; ++s)
      if (s < n_streams) old[s] = x[(size_t)s * stream_stride + e];
    float yv = y[e];
    if (scale) yv *= scale[e % width];
#pragma unroll
    for (int j = 0; j < ST_MAX_STREAMS; ++j) {
      if (j < n_streams) {
        float v = out_coef[j] * yv;
#pragma unroll
        for (int s = 0; s < ST_MAX_STREAMS; ++s)
          if (s < n_streams) v = fmaf(mix[s * n_streams + j], old[s], v);
        x[(size_t)j * stream_stride + e] = v;
      }
    }
  }
}

extern "C" int rb_streams_update(float* x, int n_streams, long long stream_stride, const float* mix, const float* out_coef,
                                 const float* y, const float* scale, int n_tokens, int width, void* stream) {
  RB_RECORDED(rb_streams_update(x, n_streams, stream_stride, mix, out_coef, y, scale, n_tokens, width, stream));
  RB_REQUIRE(n_tokens >= 0 && width > 0, "rb_streams_update: bad sizes %d x %d", n_tokens, width);
  RB_REQUIRE(n_streams >= 1 && n_streams <= ST_MAX_STREAMS && stream_stride >= 0, "rb_streams_update: %d streams (1 to %d)",
             n_streams, ST_MAX_STREAMS);
  if (n_tokens == 0) return 0;
  const size_t n = (size_t)n_tokens * width;
  const size_t blocks = (n + 255) / 256;
  streams_update_kernel<<<(int)(blocks < 65535 ? blocks : 65535), 256, 0, (hipStream_t)stream>>>(
      x, n_streams, (size_t)stream_stride, mix, out_coef, y, scale, width, n);
  RB_LAUNCH_CHECK();
  return 0;
}

// x[s][t, :] = table[ids[t], :] for every copy s.
template <typename T>
__global__ void embed_streams_kernel(const T* __restrict__ table, const int32_t* __restrict__ ids, float* __restrict__ x,
                                     int n_streams, size_t stream_stride, int width) {
  const int t = blockIdx.x;
  const T* row = table + (size_t)ids[t] * width;
  for (int j = threadIdx.x; j < width; j += blockDim.x) {
    const float v = Num<T>::load(row + j);
    for (int s = 0; s < n_streams; ++s) x[(size_t)s * stream_stride + (size_t)t * width + j] = v;
  }
}

extern "C" int rb_embed_streams(const void* table, int table_dtype, const int32_t* ids, float* x, int n_streams,
                                long long stream_stride, int n_tokens, int width, void* stream) {
  RB_RECORDED(rb_embed_streams(table, table_dtype, ids, x, n_streams, stream_stride, n_tokens, width, stream));
  RB_REQUIRE(n_tokens >= 0 && width > 0 && n_streams >= 1, "rb_embed_streams: bad sizes");
  if (n_tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  if (table_dtype == RB_F32)
    embed_streams_kernel<float><<<n_tokens, 256, 0, s>>>((const float*)table, ids, x, n_streams, (size_t)stream_stride, width);
  else if (table_dtype == RB_BF16)
    embed_streams_kernel<bf16_t><<<n_tokens, 256, 0, s>>>((const bf16_t*)table, ids, x, n_streams, (size_t)stream_stride, width);
  else
    RB_REQUIRE(false, "rb_embed_streams: unknown dtype %d", table_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}

// The same with what a model may do to an embedding's row: x[s][t, :] = table[ids[t], :] * scale + wave(pos[t]), where number 2i of
// wave(p) is sin(p inv[i]) and number 2i + 1 is cos(p inv[i]) (inv float64 [(width + 1) / 2]; null: no wave).  The angle is
// made and brought into one turn in float64, so that a late position's sine is as good as an early one's.
template <typename T>
__global__ void embed_streams_waves_kernel(const T* __restrict__ table, const int32_t* __restrict__ ids, float scale,
                                           const double* __restrict__ inv, const int32_t* __restrict__ tok_pos, float* __restrict__ x,
                                           int n_streams, size_t stream_stride, int width) {
  const int t = blockIdx.x;
  const T* row = table + (size_t)ids[t] * width;
  const double pos = (double)tok_pos[t];
  const int n_pairs = (width + 1) / 2;
  for (int i = threadIdx.x; i < n_pairs; i += blockDim.x) {
    float sn = 0.f, cs = 0.f;
    if (inv) {
      const double angle = pos * inv[i];
      const double turns = rint(angle * 0.15915494309189535);
      sincosf((float)fma(-turns, 6.283185307179586, angle), &sn, &cs);
    }
    const float a = fmaf(Num<T>::load(row + 2 * i), scale, sn);
    const bool two = 2 * i + 1 < width;
    const float b = two ? fmaf(Num<T>::load(row + 2 * i + 1), scale, cs) : 0.f;
    const bool pair = two && width % 2 == 0 && stream_stride % 2 == 0 && (reinterpret_cast<uintptr_t>(x) & 7) == 0;
    for (int s = 0; s < n_streams; ++s) {
      float* xr = x + (size_t)s * stream_stride + (size_t)t * width + 2 * i;
      if (pair) {
        *reinterpret_cast<float2*>(xr) = make_float2(a, b);
        continue;
      }
      xr[0] = a;
      if (two) xr[1] = b;
    }
  }
}

extern "C" int rb_embed_streams_waves(const void* table, int table_dtype, const int32_t* ids, float scale, const double* inv,
                                      const int32_t* tok_pos, float* x, int n_streams, long long stream_stride, int n_tokens, int width,
                                      void* stream) {
  RB_RECORDED(rb_embed_streams_waves(table, table_dtype, ids, scale, inv, tok_pos, x, n_streams, stream_stride, n_tokens, width, stream));
  RB_REQUIRE(n_tokens >= 0 && width > 0 && n_streams >= 1 && stream_stride >= 0, "rb_embed_streams_waves: bad sizes");
  RB_REQUIRE(inv == nullptr || tok_pos != nullptr, "rb_embed_streams_waves: a wave needs the tokens' positions");
  if (n_tokens == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  if (table_dtype == RB_F32)
    embed_streams_waves_kernel<float><<<n_tokens, 256, 0, s>>>((const float*)table, ids, scale, inv, tok_pos, x, n_streams,
                                                               (size_t)stream_stride, width);
  else if (table_dtype == RB_BF16)
    embed_streams_waves_kernel<bf16_t><<<n_tokens, 256, 0, s>>>((const bf16_t*)table, ids, scale, inv, tok_pos, x, n_streams,
                                                                (size_t)stream_stride, width);
  else
    RB_REQUIRE(false, "rb_embed_streams_waves: unknown dtype %d", table_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- RMS norm of a stream in several copies
// out[r] = u / sqrt(mean(u^2) + eps) * gain, u = sum_s coef[s] x[s][src], src = rows ? rows[r] : r (coef null: the plain sum).
// With an update that was still to be done (mix not null) the copies are first rebuilt from all the old ones,
//   x[t] <- sum_s mix[s, t] x[s] + out_coef[t] * y,
// in the same pass; with rows the copies stay as they are (nobody reads them again).  y of a row is a sum of terms:
//   y = sum_k (weights ? weights[src * n_terms + k] : 1) y[src * row_stride + k * term_stride]  +  sum_k extra[src * width + k * extra_stride]
// (the K slices of a product; the outputs of a token's experts and what a shared expert adds).  NS copies, or, NS 0, n_streams.
struct StreamsNormArgs {
  int n_streams;
  size_t stream_stride;
  int n_terms;
  size_t term_stride, row_stride;
  int n_extra;
  size_t extra_stride;
  float eps;
  int width;
};
template <int V>
struct Piece {
  float v[V];
};
template <int V>
__device__ __forceinline__ Piece<V> load_piece(const float* p) {
  Piece<V> r;
  if (V == 4) {
    const float4 q = ld4(p);
    r.v[0] = q.x;
    r.v[V > 1 ? 1 : 0] = q.y;
    r.v[V > 2 ? 2 : 0] = q.z;
    r.v[V - 1] = q.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V>
__device__ __forceinline__ void store_piece_f32(float* p, const Piece<V>& r) {
  if (V == 4) st4(p, r.v[0], r.v[V > 1 ? 1 : 0], r.v[V > 2 ? 2 : 0], r.v[V - 1]);
  else *p = r.v[0];
}
template <int V>
__device__ __forceinline__ void add_terms(Piece<V>& acc, const float* p, int n_terms, size_t stride, const float* w) {
  int k = 0;
  for (; k + 3 < n_terms; k += 4) {                 // four terms in flight
    Piece<V> e[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) e[u] = load_piece<V>(p + (size_t)(k + u) * stride);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float f = w ? w[k + u] : 1.0f;
#pragma unroll
      for (int i = 0; i < V; ++i) acc.v[i] = fmaf(f, e[u].v[i], acc.v[i]);
    }
  }
  for (; k < n_terms; ++k) {
    const Piece<V> e = load_piece<V>(p + (size_t)k * stride);
    const float f = w ? w[k] : 1.0f;
#pragma unroll
    for (int i = 0; i < V; ++i) acc.v[i] = fmaf(f, e.v[i], acc.v[i]);
  }
}

template <typename TO, int V, int NS>
__global__ __launch_bounds__(1024) void streams_rmsnorm_kernel(StreamsNormArgs p, float* __restrict__ x, const float* __restrict__ mix,
                                                               const float* __restrict__ out_coef, const float* __restrict__ y,
                                                               const float* __restrict__ weights, const float* __restrict__ extra,
                                                               const float* __restrict__ coef, const float* __restrict__ gain,
                                                               const int32_t* __restrict__ rows, TO* __restrict__ out) {
  extern __shared__ float u[];
  __shared__ float scratch[16];
  constexpr int MOST = NS > 0 ? NS : ST_MAX_STREAMS;
  const int n = NS > 0 ? NS : p.n_streams;
  const int r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : (size_t)r;
  const bool write_back = mix != nullptr && rows == nullptr;
  float ss = 0.f;
  for (int j = V * threadIdx.x; j < p.width; j += V * blockDim.x) {
    Piece<V> old[MOST], v, yv;
#pragma unroll
    for (int s = 0; s < MOST; ++s)
      if (s < n) old[s] = load_piece<V>(x + (size_t)s * p.stream_stride + src * p.width + j);
#pragma unroll
    for (int i = 0; i < V; ++i) v.v[i] = yv.v[i] = 0.f;
    if (mix) {
      add_terms<V>(yv, y + src * p.row_stride + j, p.n_terms, p.term_stride, weights ? weights + src * p.n_terms : nullptr);
      if (extra) add_terms<V>(yv, extra + src * p.width + j, p.n_extra, p.extra_stride, nullptr);
#pragma unroll
      for (int t = 0; t < MOST; ++t) {
        if (t < n) {
          const float oc = out_coef[t], ic = coef ? coef[t] : 1.0f;
          Piece<V> nv;
#pragma unroll
          for (int i = 0; i < V; ++i) nv.v[i] = oc * yv.v[i];
#pragma unroll
          for (int s = 0; s < MOST; ++s)
            if (s < n) {
              const float m = mix[s * n + t];
#pragma unroll
              for (int i = 0; i < V; ++i) nv.v[i] = fmaf(m, old[s].v[i], nv.v[i]);
            }
          if (write_back) store_piece_f32<V>(x + (size_t)t * p.stream_stride + src * p.width + j, nv);
#pragma unroll
          for (int i = 0; i < V; ++i) v.v[i] = fmaf(ic, nv.v[i], v.v[i]);
        }
      }
    } else {
#pragma unroll
      for (int s = 0; s < MOST; ++s)
        if (s < n) {
          const float ic = coef ? coef[s] : 1.0f;
#pragma unroll
          for (int i = 0; i < V; ++i) v.v[i] = fmaf(ic, old[s].v[i], v.v[i]);
        }
    }
    store_piece_f32<V>(u + j, v);
#pragma unroll
    for (int i = 0; i < V; ++i) ss = fmaf(v.v[i], v.v[i], ss);
  }
  // the gain of this thread's first numbers is asked for now, so that it arrives under the reduction
  const int j0 = V * threadIdx.x;
  Piece<V> g0;
#pragma unroll
  for (int i = 0; i < V; ++i) g0.v[i] = 0.f;
  if (j0 < p.width) g0 = load_piece<V>(gain + j0);
  __builtin_amdgcn_sched_barrier(0);
  const float f = 1.0f / sqrtf(block_sum(ss, scratch) / (float)p.width + p.eps);
  TO* orow = out + (size_t)r * p.width;
  for (int j = j0; j < p.width; j += V * blockDim.x) {
    const Piece<V> v = load_piece<V>(u + j), g = j == j0 ? g0 : load_piece<V>(gain + j);
    if (V == 4)
      st4(orow + j, v.v[0] * f * g.v[0], v.v[V > 1 ? 1 : 0] * f * g.v[V > 1 ? 1 : 0], v.v[V > 2 ? 2 : 0] * f * g.v[V > 2 ? 2 : 0],
          v.v[V - 1] * f * g.v[V - 1]);
    else
      Num<TO>::store(orow + j, v.v[0] * f * g.v[0]);
  }
}

extern "C" int rb_streams_rmsnorm(float* x, int n_streams, long long stream_stride, const float* mix, const float* out_coef, const float* y,
                                  int n_terms, long long term_stride, long long row_stride, const float* weights, const float* extra,
                                  int n_extra, long long extra_stride, const float* coef, const float* gain, float eps,
                                  const int32_t* rows, int n_rows, int width, void* out, int out_dtype, void* stream) {
  RB_RECORDED(rb_streams_rmsnorm(x, n_streams, stream_stride, mix, out_coef, y, n_terms, term_stride, row_stride, weights, extra, n_extra,
                                 extra_stride, coef, gain, eps, rows, n_rows, width, out, out_dtype, stream));
  RB_REQUIRE(n_rows >= 0 && width > 0 && width <= 16384, "rb_streams_rmsnorm: bad sizes %d x %d (width at most 16384)", n_rows, width);
  RB_REQUIRE(n_streams >= 1 && n_streams <= ST_MAX_STREAMS && stream_stride >= 0, "rb_streams_rmsnorm: %d streams (1 to %d)", n_streams,
             ST_MAX_STREAMS);
  RB_REQUIRE(mix == nullptr || (out_coef != nullptr && y != nullptr && n_terms >= 1 && term_stride >= 0 && row_stride >= width),
             "rb_streams_rmsnorm: an update needs out_coef and the terms of y");
  RB_REQUIRE(extra == nullptr || (mix != nullptr && n_extra >= 1 && extra_stride >= 0), "rb_streams_rmsnorm: more terms go with an update");
  RB_REQUIRE(out_dtype == RB_F32 || out_dtype == RB_BF16, "rb_streams_rmsnorm: unknown dtype %d", out_dtype);
  if (n_rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const size_t lds = (size_t)width * sizeof(float);
  auto aligned = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  const bool vec = width % 4 == 0 && stream_stride % 4 == 0 && term_stride % 4 == 0 && row_stride % 4 == 0 && extra_stride % 4 == 0 &&
                   aligned(x) && aligned(y) && aligned(extra) && aligned(gain) && aligned(out);
  const StreamsNormArgs p = {n_streams, (size_t)stream_stride, n_terms, (size_t)term_stride, (size_t)row_stride, n_extra,
                             (size_t)extra_stride, eps, width};
  int threads = vec ? ((width / 4 + RB_WAVE - 1) / RB_WAVE) * RB_WAVE : 256;
  if (threads > 1024) threads = 1024;
#define ST_GO(TO, V, NS) \
  streams_rmsnorm_kernel<TO, V, NS><<<n_rows, threads, lds, s>>>(p, x, mix, out_coef, y, weights, extra, coef, gain, rows, (TO*)out)
#define ST_BY_COPIES(TO)                    \
  do {                                      \
    if (!vec) ST_GO(TO, 1, 0);              \
    else if (n_streams == 1) ST_GO(TO, 4, 1); \
    else if (n_streams == 2) ST_GO(TO, 4, 2); \
    else if (n_streams == 3) ST_GO(TO, 4, 3); \
    else if (n_streams == 4) ST_GO(TO, 4, 4); \
    else ST_GO(TO, 4, 0);                   \
  } while (0)
  if (out_dtype == RB_F32) ST_BY_COPIES(float);
  else ST_BY_COPIES(bf16_t);
#undef ST_BY_COPIES
#undef ST_GO
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- xIELU
// z > 0: softplus(p) z^2 + z / 2;  z <= 0: (1/2 + softplus(q)) (exp(z) - 1 - z) + z / 2, with (p, q) = act[0..1].
__device__ __forceinline__ void xielu_store4(float* p, float a, float b, float c, float d) {
  *reinterpret_cast<float4*>(p) = make_float4(a, b, c, d);
}
__device__ __forceinline__ void xielu_store4(bf16_t* p, float a, float b, float c, float d) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
}

// four values a thread with 16-byte loads (n4 quads), then the rest one by one
template <typename TO>
__global__ void xielu_kernel(const float* __restrict__ z, const float* __restrict__ act, TO* __restrict__ out, size_t n) {
  const XieluPair pair = xielu_pair(act);
  const float ap = pair.ap, an = pair.an;
  const size_t n4 = n / 4;
  for (size_t e = (size_t)blockIdx.x * blockDim.x + threadIdx.x; e < n4; e += (size_t)gridDim.x * blockDim.x) {
    const float4 v = *reinterpret_cast<const float4*>(z + 4 * e);
    xielu_store4(out + 4 * e, xielu_value(v.x, ap, an), xielu_value(v.y, ap, an), xielu_value(v.z, ap, an),
                 xielu_value(v.w, ap, an));
  }
  for (size_t e = 4 * n4 + (size_t)blockIdx.x * blockDim.x + threadIdx.x; e < n; e += (size_t)gridDim.x * blockDim.x)
    Num<TO>::store(out + e, xielu_value(z[e], ap, an));
}

extern "C" int rb_xielu(const float* z, const float* act, void* out, int out_dtype, long long n, void* stream) {
  RB_RECORDED(rb_xielu(z, act, out, out_dtype, n, stream));
  RB_REQUIRE(n >= 0, "rb_xielu: bad size");
  if (n == 0) return 0;
  const size_t blocks = ((size_t)n / 4 + 255) / 256 + 1;
  const int grid = (int)(blocks < 65535 ? blocks : 65535);
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == RB_F32)
    xielu_kernel<float><<<grid, 256, 0, s>>>(z, act, (float*)out, (size_t)n);
  else if (out_dtype == RB_BF16)
    xielu_kernel<bf16_t><<<grid, 256, 0, s>>>(z, act, (bf16_t*)out, (size_t)n);
  else
    RB_REQUIRE(false, "rb_xielu: unknown dtype %d", out_dtype);
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- cap of the logits
// x <- cap * tanh(x / cap), in place.
__global__ void tanh_cap_kernel(float* __restrict__ x, float cap, size_t n) {
  for (size_t e = (size_t)blockIdx.x * blockDim.x + threadIdx.x; e < n; e += (size_t)gridDim.x * blockDim.x)
    x[e] = cap * tanhf(x[e] / cap);
}

extern "C" int rb_tanh_cap(float* x, float cap, long long n, void* stream) {
  RB_RECORDED(rb_tanh_cap(x, cap, n, stream));
  RB_REQUIRE(n >= 0 && cap > 0.f, "rb_tanh_cap: bad size or cap");
  if (n == 0) return 0;
  const size_t blocks = ((size_t)n + 255) / 256;
  tanh_cap_kernel<<<(int)(blocks < 65535 ? blocks : 65535), 256, 0, (hipStream_t)stream>>>(x, cap, (size_t)n);
  RB_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------- a norm that is an element-wise tanh
// norm(v) = tanh(alpha v) w + b, number by number (alpha one number, w and b a row).  In one pass over the rows:
//   v = x[src] + after(y[src]);  without rows x[src] = v;  out[r] = before(v),    src = rows ? rows[r] : r
// where after is the norm on a sublayer's output (a1, w1, b1; a1 null: y is added as it is) and before the one in front of the
// next sublayer (a2, w2, b2; out null: none).  y is a sum of n_terms terms, term_stride floats apart, a row of them row_stride
// apart (K slices of a product, or the outputs of a token's experts), term k times weights[src * n_terms + k] where given;
// y null: nothing is added.  A thread keeps the parameters of its columns and walks rows.
struct TanhNormArgs {
  float* x;
  const float* y;
  int n_terms;
  size_t term_stride, row_stride;
  const float* weights;
  const float *a1, *w1, *b1, *a2, *w2, *b2;
  const int32_t* rows;
  int n_rows, width;
};

// tanh on the hardware's exponential and reciprocal: (1 - e) / (1 + e) with e = exp(-2 |z|), within 2e-7 of the function
__device__ __forceinline__ float tanh_fast(float z) {
  const float e = __builtin_amdgcn_exp2f(-2.8853900817779268f * fabsf(z));
  return copysignf((1.0f - e) * __builtin_amdgcn_rcpf(1.0f + e), z);
}
template <typename TO>
__device__ __forceinline__ float tanh_norm_value(float z) { return tanh_fast(z); }
template <>
__device__ __forceinline__ float tanh_norm_value<float>(float z) { return tanhf(z); }

template <typename TO, int V>
__global__ __launch_bounds__(256) void tanh_norm_kernel(TanhNormArgs p, TO* __restrict__ out) {
  const int j = V * (blockIdx.x * blockDim.x + threadIdx.x);
  if (j >= p.width) return;
  float w1[V], b1[V], w2[V], b2[V];
  const float a1 = p.a1 ? *p.a1 : 0.f, a2 = p.a2 ? *p.a2 : 0.f;
  auto load = [&](float* d, const float* s) {
    if (V == 4) {
      const float4 v = ld4(s);
      d[0] = v.x;
      d[V > 1 ? 1 : 0] = v.y;
      d[V > 2 ? 2 : 0] = v.z;
      d[V - 1] = v.w;
    } else {
      d[0] = *s;
    }
  };
  if (p.a1) {
    load(w1, p.w1 + j);
    load(b1, p.b1 + j);
  }
  if (out) {
    load(w2, p.w2 + j);
    load(b2, p.b2 + j);
  }
  for (int r = blockIdx.y; r < p.n_rows; r += gridDim.y) {
    const size_t src = p.rows ? (size_t)p.rows[r] : (size_t)r;
    float v[V];
    load(v, p.x + src * p.width + j);
    if (p.y) {
      const float* yp = p.y + src * p.row_stride + j;
      const float* wp = p.weights ? p.weights + src * p.n_terms : nullptr;
      float acc[V];
#pragma unroll
      for (int i = 0; i < V; ++i) acc[i] = 0.f;
      int k = 0;
      for (; k + 3 < p.n_terms; k += 4) {               // four terms in flight
        float e[4][V];
#pragma unroll
        for (int u = 0; u < 4; ++u) load(e[u], yp + (size_t)(k + u) * p.term_stride);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const float f = wp ? wp[k + u] : 1.0f;
#pragma unroll
          for (int i = 0; i < V; ++i) acc[i] = fmaf(f, e[u][i], acc[i]);
        }
      }
      for (; k < p.n_terms; ++k) {
        float e[V];
        load(e, yp + (size_t)k * p.term_stride);
        const float f = wp ? wp[k] : 1.0f;
#pragma unroll
        for (int i = 0; i < V; ++i) acc[i] = fmaf(f, e[i], acc[i]);
      }
#pragma unroll
      for (int i = 0; i < V; ++i) v[i] += p.a1 ? fmaf(tanh_norm_value<TO>(a1 * acc[i]), w1[i], b1[i]) : acc[i];
      if (!p.rows) {
        float* xd = p.x + src * p.width + j;
        if (V == 4) st4(xd, v[0], v[V > 1 ? 1 : 0], v[V > 2 ? 2 : 0], v[V - 1]);
        else *xd = v[0];
      }
    }
    if (out) {
      float o[V];
#pragma unroll
      for (int i = 0; i < V; ++i) o[i] = fmaf(tanh_norm_value<TO>(a2 * v[i]), w2[i], b2[i]);
      TO* od = out + (size_t)r * p.width + j;
      if (V == 4) st4(od, o[0], o[V > 1 ? 1 : 0], o[V > 2 ? 2 : 0], o[V - 1]);
      else Num<TO>::store(od, o[0]);
    }
  }
}

extern "C" int rb_tanh_norm(float* x, const float* y, int n_terms, long long term_stride, long long row_stride, const float* weights,
                            const float* a1, const float* w1, const float* b1, const float* a2, const float* w2, const float* b2,
                            const int32_t* rows, int n_rows, int width, void* out, int out_dtype, void* stream) {
  RB_RECORDED(rb_tanh_norm(x, y, n_terms, term_stride, row_stride, weights, a1, w1, b1, a2, w2, b2, rows, n_rows, width, out, out_dtype,
                           stream));
  RB_REQUIRE(n_rows >= 0 && width > 0 && x != nullptr, "rb_tanh_norm: bad sizes %d x %d", n_rows, width);
  RB_REQUIRE(y == nullptr || (n_terms >= 1 && term_stride >= 0 && row_stride >= width), "rb_tanh_norm: bad terms");
  RB_REQUIRE(a1 == nullptr || (w1 != nullptr && b1 != nullptr), "rb_tanh_norm: a norm needs its weight and bias");
  RB_REQUIRE(out == nullptr || (a2 != nullptr && w2 != nullptr && b2 != nullptr), "rb_tanh_norm: a norm needs its weight and bias");
  RB_REQUIRE(out != nullptr || (y != nullptr && rows == nullptr), "rb_tanh_norm: nothing to do");
  RB_REQUIRE(out_dtype == RB_F32 || out_dtype == RB_BF16, "rb_tanh_norm: unknown dtype %d", out_dtype);
  if (n_rows == 0) return 0;
  TanhNormArgs p = {x, y, n_terms, (size_t)term_stride, (size_t)row_stride, weights, a1, w1, b1, a2, w2, b2, rows, n_rows, width};
  auto aligned = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  const bool vec = width % 4 == 0 && term_stride % 4 == 0 && row_stride % 4 == 0 && aligned(x) && aligned(y) && aligned(w1) && aligned(b1) &&
                   aligned(w2) && aligned(b2) && aligned(out);
  const int cols = vec ? width / 4 : width;
  // few rows: small workgroups spread over the compute units; many: as many workgroups as keep them busy, each walking rows
  const int threads = (long long)n_rows * ((cols + 255) / 256) >= rb_compute_units() ? 256 : RB_WAVE;
  const int gx = (cols + threads - 1) / threads;
  int gy = (8 * rb_compute_units() + gx - 1) / gx;
  if (gy > n_rows) gy = n_rows;
  if (gy > 65535) gy = 65535;
  dim3 grid(gx, gy);
  hipStream_t s = (hipStream_t)stream;
  if (out_dtype == RB_F32) {
    if (vec) tanh_norm_kernel<float, 4><<<grid, threads, 0, s>>>(p, (float*)out);
    else tanh_norm_kernel<float, 1><<<grid, threads, 0, s>>>(p, (float*)out);
  } else {
    if (vec) tanh_norm_kernel<bf16_t, 4><<<grid, threads, 0, s>>>(p, (bf16_t*)out);
    else tanh_norm_kernel<bf16_t, 1><<<grid, threads, 0, s>>>(p, (bf16_t*)out);
  }
  RB_LAUNCH_CHECK();
  return 0;
}
