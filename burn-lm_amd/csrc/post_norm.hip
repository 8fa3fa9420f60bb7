// Sublayer results that are normed before they join the residual, and what follows the join, as one kernel per row:
//
//   y_i = y_i + (bias_i ? bias_i : 0)                                   a last projection's bias
//   y = sum_i scale_i * (gamma_i ? n(y_i, eps_i) * gamma_i : y_i)       up to two results (two mixers side by side)
//   y = post_gamma ? n(y, post_eps) * post_gamma : y                    the norm behind the sublayer
//   v = (fresh ? 0 : h[r]) + (vec ? vec : 0) + y                        fresh: the residual starts anew from y
//   h[r] = v if write_h
//   out[i] = gamma ? n(v, eps) * gamma : v                              the next sublayer's input, rounded once
//
// with n(x, eps) = x / sqrt(mean(x^2) + eps) and r = rows ? rows[i] : i.  A result y_i is [T][D] in either kernel
// type, or float planes [P][T][D] that are summed (partial products of a matrix product whose K was cut).  All sums,
// norms and the residual are float; out rows are ldo elements apart, so that they can be one half of wider rows.
//
// Also here: rows of the embedding with the positions' vectors added.
#include "common.h"

struct PnTerm {
  const void* y;
  const float* gamma;
  const float* bias;
  size_t stride;      // elements between planes
  int planes, dtype;
  float scale, eps;
};
struct PnArgs {
  PnTerm term[2];
  const float* post_gamma;
  const float* vec;
  const float* gamma;
  const int* rows;
  float post_eps, eps;
  int n_terms, fresh, write_h, D, ldo;
};

__device__ __forceinline__ void pn_load4(const float* p, float* v) {
  const float4 r = *reinterpret_cast<const float4*>(p);
  v[0] = r.x; v[1] = r.y; v[2] = r.z; v[3] = r.w;
}
__device__ __forceinline__ void pn_store4(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void pn_store4(bf16* p, const float* v) {
  uint2 r;
  r.x = f32x2_to_bf16x2_bits(v[0], v[1]);
  r.y = f32x2_to_bf16x2_bits(v[2], v[3]);
  *reinterpret_cast<uint2*>(p) = r;
}

// four channels of a result, its planes summed in order (four planes' loads under way at a time)
__device__ __forceinline__ void pn_result4(const PnTerm& t, size_t at, float* v) {
  if (t.dtype == BLM_BF16) {
    const uint2 r = *reinterpret_cast<const uint2*>(reinterpret_cast<const bf16*>(t.y) + at);
    v[0] = __uint_as_float(r.x << 16); v[1] = __uint_as_float(r.x & 0xffff0000u);
    v[2] = __uint_as_float(r.y << 16); v[3] = __uint_as_float(r.y & 0xffff0000u);
    return;
  }
  const float* y = reinterpret_cast<const float*>(t.y) + at;
  if (t.planes == 1) { pn_load4(y, v); return; }
  v[0] = v[1] = v[2] = v[3] = 0.f;
  for (int p0 = 0; p0 < t.planes; p0 += 4) {
    float a[4][4];
#pragma unroll
    for (int q = 0; q < 4; ++q) pn_load4(y + (size_t)min(p0 + q, t.planes - 1) * t.stride, a[q]);
#pragma unroll
    for (int q = 0; q < 4; ++q)
      if (p0 + q < t.planes) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] += a[q][e];
      }
  }
}
__device__ __forceinline__ float pn_result1(const PnTerm& t, size_t at, int d) {
  float v = t.bias ? t.bias[d] : 0.f;
  if (t.dtype == BLM_BF16) return v + to_float(reinterpret_cast<const bf16*>(t.y)[at]);
  const float* y = reinterpret_cast<const float*>(t.y) + at;
  for (int p = 0; p < t.planes; ++p) v += y[(size_t)p * t.stride];
  return v;
}

// sums of two values over the block at once; red holds 2 * 16 floats and must be free
__device__ __forceinline__ void pn_block_sum2(float& a, float& b, float* red) {
  const int lane = threadIdx.x & (BLM_WAVE - 1), w = threadIdx.x / BLM_WAVE, nw = blockDim.x / BLM_WAVE;
  a = wave_sum(a);
  b = wave_sum(b);
  if (nw == 1) return;
  if (lane == 0) { red[w] = a; red[16 + w] = b; }
  __syncthreads();
  a = red[0];
  b = red[16];
  for (int k = 1; k < nw; ++k) { a += red[k]; b += red[16 + k]; }
}

// Rows that fit the block's registers (D a multiple of 4, at most 4 * blockDim * ITERS): one pass over memory.
template <typename TA, int ITERS, int NT>
__global__ void __launch_bounds__(512) post_norm_vec_kernel(float* __restrict__ h, TA* __restrict__ out, PnArgs g) {
  __shared__ float red[3][32];
  const int i = blockIdx.x, D = g.D;
  const int r = g.rows ? g.rows[i] : i;
  float* hr = h + (size_t)r * D;
  const size_t row = (size_t)r * D;
  // everything the row needs is asked for at once: results, residual, weights
  float y[NT][ITERS][4], v[ITERS][4], w[NT][ITERS][4], wp[ITERS][4], wo[ITERS][4];
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int d = (it * blockDim.x + threadIdx.x) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[it][e] = 0.f; wp[it][e] = 1.f; wo[it][e] = 1.f;
#pragma unroll
      for (int n = 0; n < NT; ++n) { y[n][it][e] = 0.f; w[n][it][e] = 1.f; }
    }
    if (d < D) {
      if (!g.fresh) pn_load4(hr + d, v[it]);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        pn_result4(g.term[n], row + d, y[n][it]);
        if (g.term[n].bias) {
          float x[4];
          pn_load4(g.term[n].bias + d, x);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[n][it][e] += x[e];
        }
        if (g.term[n].gamma) pn_load4(g.term[n].gamma + d, w[n][it]);
      }
      if (g.post_gamma) pn_load4(g.post_gamma + d, wp[it]);
      if (g.gamma) pn_load4(g.gamma + d, wo[it]);
      if (g.vec) {
        float x[4];
        pn_load4(g.vec + d, x);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[it][e] += x[e];
      }
    }
  }
  float c[2] = {g.term[0].scale, g.term[1].scale};
  if (g.term[0].gamma || (NT == 2 && g.term[1].gamma)) {
    float ss[2] = {0.f, 0.f};
#pragma unroll
    for (int it = 0; it < ITERS; ++it)
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int n = 0; n < NT; ++n) ss[n] = fmaf(y[n][it][e], y[n][it][e], ss[n]);
    pn_block_sum2(ss[0], ss[1], red[0]);
#pragma unroll
    for (int n = 0; n < NT; ++n)
      if (g.term[n].gamma) c[n] /= sqrtf(ss[n] / (float)D + g.term[n].eps);
  }
  float sy = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float a = y[0][it][e] * c[0] * w[0][it][e];
      if (NT == 2) a = fmaf(y[NT - 1][it][e] * c[1], w[NT - 1][it][e], a);
      y[0][it][e] = a;
      sy = fmaf(a, a, sy);
    }
  float cp = 1.f;
  if (g.post_gamma) cp = 1.0f / sqrtf(block_sum<true>(sy, red[1]) / (float)D + g.post_eps);
  float sv = 0.f;
#pragma unroll
  for (int it = 0; it < ITERS; ++it)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[it][e] += y[0][it][e] * cp * wp[it][e];
      sv = fmaf(v[it][e], v[it][e], sv);
    }
  float co = 1.f;
  if (g.gamma) co = 1.0f / sqrtf(block_sum<true>(sv, red[2]) / (float)D + g.eps);
#pragma unroll
  for (int it = 0; it < ITERS; ++it) {
    const int d = (it * blockDim.x + threadIdx.x) * 4;
    if (d < D) {
      if (g.write_h) pn_store4(hr + d, v[it]);
      if (out) {
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = v[it][e] * co * wo[it][e];
        pn_store4(out + (size_t)i * g.ldo + d, o);
      }
    }
  }
}

// Any width: the row is walked once per norm, results read again each time.
template <typename TA>
__global__ void __launch_bounds__(256) post_norm_kernel(float* __restrict__ h, TA* __restrict__ out, PnArgs g) {
  __shared__ float red[3][32];
  const int i = blockIdx.x, D = g.D;
  const int r = g.rows ? g.rows[i] : i;
  float* hr = h + (size_t)r * D;
  const size_t row = (size_t)r * D;
  float c[2] = {g.term[0].scale, g.term[1].scale};
  if (g.term[0].gamma || (g.n_terms == 2 && g.term[1].gamma)) {
    float ss[2] = {0.f, 0.f};
    for (int d = threadIdx.x; d < D; d += blockDim.x)
      for (int n = 0; n < g.n_terms; ++n) {
        const float a = pn_result1(g.term[n], row + d, d);
        ss[n] = fmaf(a, a, ss[n]);
      }
    pn_block_sum2(ss[0], ss[1], red[0]);
    for (int n = 0; n < g.n_terms; ++n)
      if (g.term[n].gamma) c[n] /= sqrtf(ss[n] / (float)D + g.term[n].eps);
  }
  auto sum_of = [&](int d) {
    float a = 0.f;
    for (int n = 0; n < g.n_terms; ++n) a = fmaf(pn_result1(g.term[n], row + d, d) * c[n], g.term[n].gamma ? g.term[n].gamma[d] : 1.f, a);
    return a;
  };
  float cp = 1.f;
  if (g.post_gamma) {
    float sy = 0.f;
    for (int d = threadIdx.x; d < D; d += blockDim.x) { const float a = sum_of(d); sy = fmaf(a, a, sy); }
    cp = 1.0f / sqrtf(block_sum<true>(sy, red[1]) / (float)D + g.post_eps);
  }
  auto joined = [&](int d) {
    return (g.fresh ? 0.f : hr[d]) + (g.vec ? g.vec[d] : 0.f) + sum_of(d) * cp * (g.post_gamma ? g.post_gamma[d] : 1.f);
  };
  float co = 1.f;
  if (g.gamma) {
    float sv = 0.f;
    for (int d = threadIdx.x; d < D; d += blockDim.x) { const float v = joined(d); sv = fmaf(v, v, sv); }
    co = 1.0f / sqrtf(block_sum<true>(sv, red[2]) / (float)D + g.eps);
  }
  for (int d = threadIdx.x; d < D; d += blockDim.x) {
    const float v = joined(d);      // the thread's own channel: h is not written before its last read
    if (g.write_h) hr[d] = v;
    if (out) out[(size_t)i * g.ldo + d] = from_float<TA>(v * co * (g.gamma ? g.gamma[d] : 1.f));
  }
}

// Terms: y, dtype, planes, plane stride, scale, gamma (or null), eps, bias (or null); the second one may have a null y (one term).
// out may be null (the residual alone), gamma null (out is the residual's rows as they are).
extern "C" int blm_post_norm(float* h, const void* y0, int dtype0, int planes0, long long stride0, float scale0, const float* gamma0,
                             float eps0, const float* bias0, const void* y1, int dtype1, int planes1, long long stride1, float scale1,
                             const float* gamma1, float eps1, const float* bias1, const float* post_gamma, float post_eps, int fresh,
                             const float* vec, int write_h, const float* gamma, float eps, void* out, int act_dtype, int ldo,
                             const int* rows, int n_out, int D, hipStream_t stream) {
  BLM_REQUIRE(h && n_out > 0 && D > 0 && y0 && (out || write_h), "post_norm: bad sizes n=%d D=%d, or nothing to write", n_out, D);
  BLM_REQUIRE(!out || ldo >= D, "post_norm: rows of %d elements do not hold %d", ldo, D);
  PnArgs g;
  g.term[0] = PnTerm{y0, gamma0, bias0, (size_t)stride0, planes0, dtype0, scale0, eps0};
  g.term[1] = PnTerm{y1, gamma1, bias1, (size_t)stride1, planes1, dtype1, scale1, eps1};
  g.n_terms = y1 ? 2 : 1;
  if (!y1) g.term[1] = PnTerm{y0, nullptr, nullptr, 0, 1, dtype0, 0.f, 0.f};
  for (int n = 0; n < g.n_terms; ++n)
    BLM_REQUIRE(g.term[n].planes >= 1 && (g.term[n].dtype == BLM_F32 || (g.term[n].dtype == BLM_BF16 && g.term[n].planes == 1)),
                "post_norm: result %d is not float planes or one bfloat16 plane", n);
  BLM_REQUIRE(!out || act_dtype == BLM_F32 || act_dtype == BLM_BF16, "post_norm: unsupported dtype %d", act_dtype);
  g.post_gamma = post_gamma; g.vec = vec; g.gamma = gamma; g.rows = rows;
  g.post_eps = post_eps; g.eps = eps;
  g.fresh = fresh; g.write_h = write_h; g.D = D; g.ldo = ldo;
  const int esize = act_dtype == BLM_F32 ? 4 : 2;
  bool vec4 = D % 4 == 0 && ((uintptr_t)h & 15) == 0 && (!out || (((uintptr_t)out & (4 * esize - 1)) == 0 && ldo % 4 == 0)) &&
              (((uintptr_t)post_gamma | (uintptr_t)vec | (uintptr_t)gamma) & 15) == 0;
  for (int n = 0; n < g.n_terms; ++n)
    vec4 = vec4 && ((uintptr_t)g.term[n].y & (g.term[n].dtype == BLM_F32 ? 15 : 7)) == 0 && (((uintptr_t)g.term[n].gamma | (uintptr_t)g.term[n].bias) & 15) == 0 &&
           g.term[n].stride % 4 == 0;
  const int threads = D >= 2048 ? 512 : 256;
  if (vec4 && D <= threads * 16) {
    const int iters = (D + 4 * threads - 1) / (4 * threads);
#define PN_RUN(TA, IT, NT) hipLaunchKernelGGL((post_norm_vec_kernel<TA, IT, NT>), dim3(n_out), dim3(threads), 0, stream, h, (TA*)out, g)
#define PN_PICK(TA, NT) do { if (iters == 1) PN_RUN(TA, 1, NT); else if (iters == 2) PN_RUN(TA, 2, NT); else PN_RUN(TA, 4, NT); } while (0)
    if (act_dtype == BLM_F32) { if (y1) PN_PICK(float, 2); else PN_PICK(float, 1); }
    else { if (y1) PN_PICK(bf16, 2); else PN_PICK(bf16, 1); }
#undef PN_PICK
#undef PN_RUN
    BLM_LAUNCH_CHECK("post_norm_vec");
    return 0;
  }
  if (act_dtype == BLM_F32) hipLaunchKernelGGL(post_norm_kernel<float>, dim3(n_out), dim3(256), 0, stream, h, (float*)out, g);
  else hipLaunchKernelGGL(post_norm_kernel<bf16>, dim3(n_out), dim3(256), 0, stream, h, (bf16*)out, g);
  BLM_LAUNCH_CHECK("post_norm");
  return 0;
}

// ---------------------------------------------------------------------------------------
// h[t][2i] = table[id][2i] + sin(2 pi p_t turns[i]), h[t][2i + 1] = ... + cos(...): turns[i] (double) is the angle per
// position in full turns, so that the angle is reduced exactly before it becomes a float, at any position.  The token
// of row t: (*source)[source_rows[t]] where source_rows is given and not negative, else ids[t]; an id outside [0, V)
// gives a row of NaN.  copy (or null): the row once more in TA, rows ld_copy elements apart.
// ---------------------------------------------------------------------------------------
template <typename TW, typename TA>
__global__ void embed_positions_kernel(const TW* __restrict__ table, const int* __restrict__ ids, const int* __restrict__ source_rows,
                                       const int* const* __restrict__ source, const int* __restrict__ positions,
                                       const double* __restrict__ turns, float* __restrict__ h, TA* __restrict__ copy, int ld_copy,
                                       int D, int V) {
  const int t = blockIdx.x;
  const int sr = source_rows ? source_rows[t] : -1;
  const int id = sr >= 0 ? (*source)[sr] : ids[t];
  float* out = h + (size_t)t * D;
  TA* c = copy ? copy + (size_t)t * ld_copy : nullptr;
  const bool bad = (unsigned)id >= (unsigned)V;
  const TW* row = table + (size_t)(bad ? 0 : id) * D;
  const double p = (double)positions[t];
  for (int i = threadIdx.x; i < (D + 1) / 2; i += blockDim.x) {
    float add[2] = {0.f, 0.f};
    if (turns) {
      const double a = p * turns[i];
      sincospif(2.0f * (float)(a - rint(a)), &add[0], &add[1]);
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int d = 2 * i + e;
      if (d < D) {
        const float v = bad ? __builtin_nanf("") : to_float(row[d]) + add[e];
        out[d] = v;
        if (c) c[d] = from_float<TA>(v);
      }
    }
  }
}

extern "C" int blm_embed_positions(const void* table, int table_dtype, const int* ids, const int* source_rows, const void* source_cell,
                                   const int* positions, const double* turns, float* h, void* copy, int copy_dtype, int ld_copy,
                                   int T, int D, int V, hipStream_t stream) {
  BLM_REQUIRE(T > 0 && D > 0 && V > 0 && positions, "embed_positions: bad sizes T=%d D=%d V=%d", T, D, V);
  BLM_REQUIRE(!source_rows || (source_cell && ((size_t)source_cell & 7) == 0),
              "embed_positions: needs an 8-byte aligned cell with the tokens' address");
  BLM_REQUIRE(!copy || ld_copy >= D, "embed_positions: rows of %d elements do not hold %d", ld_copy, D);
  BLM_REQUIRE((table_dtype == BLM_F32 || table_dtype == BLM_BF16) && (!copy || copy_dtype == BLM_F32 || copy_dtype == BLM_BF16),
              "embed_positions: unsupported dtypes %d, %d", table_dtype, copy_dtype);
  const int* const* cell = (const int* const*)source_cell;
  const dim3 grid(T), block(256);
#define EP_RUN(TW, TA)                                                                                                 \
  hipLaunchKernelGGL((embed_positions_kernel<TW, TA>), grid, block, 0, stream, (const TW*)table, ids, source_rows, cell, \
                     positions, turns, h, (TA*)copy, ld_copy, D, V)
  const bool f32_copy = !copy || copy_dtype == BLM_F32;
  if (table_dtype == BLM_F32) { if (f32_copy) EP_RUN(float, float); else EP_RUN(float, bf16); }
  else { if (f32_copy) EP_RUN(bf16, float); else EP_RUN(bf16, bf16); }
#undef EP_RUN
  BLM_LAUNCH_CHECK("embed_positions");
  return 0;
}

// ---------------------------------------------------------------------------------------
// out[e] = sum over planes p of y[p][e], in order, float: the partial products of a narrow matrix product
// ---------------------------------------------------------------------------------------
__global__ void sum_planes_kernel(const float* __restrict__ y, int planes, long long n, float* __restrict__ out) {
  const long long stride = (long long)gridDim.x * blockDim.x;
  for (long long e = (long long)blockIdx.x * blockDim.x + threadIdx.x; e < n; e += stride) {
    float v = 0.f;
    for (int p0 = 0; p0 < planes; p0 += 8) {
      float a[8];
#pragma unroll
      for (int q = 0; q < 8; ++q) a[q] = y[(size_t)min(p0 + q, planes - 1) * n + e];
#pragma unroll
      for (int q = 0; q < 8; ++q)
        if (p0 + q < planes) v += a[q];
    }
    out[e] = v;
  }
}

extern "C" int blm_sum_planes(const float* y, int planes, long long n, float* out, hipStream_t stream) {
  BLM_REQUIRE(planes >= 1 && n > 0, "sum_planes: bad sizes, %d planes", planes);
  const unsigned blocks = (unsigned)((n + 255) / 256 < 65535 ? (n + 255) / 256 : 65535);
  hipLaunchKernelGGL(sum_planes_kernel, dim3(blocks), dim3(256), 0, stream, y, planes, n, out);
  BLM_LAUNCH_CHECK("sum_planes");
  return 0;
}
