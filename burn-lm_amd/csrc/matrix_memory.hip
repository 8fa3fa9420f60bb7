// Matrix memory with an exponential input gate and a forget gate per head (the mLSTM cell of xLSTM), stabilised by a
// running maximum.  Per head, with the logarithms i_t and f_t of the two gates:
//   m_t = max(f_t + m_(t-1), i_t)                                                    (m_0 = 0)
//   S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T                n_t likewise with k_t alone
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
// with i = cap tanh((z_i + b_i) / cap), f = log sigmoid(cap tanh((z_f + b_f) / cap)), q scaled by q_scale; then every
// head's o over its root mean square, times a weight per lane and the sigmoid of the output gate's logits.
// State per sequence, float: S [H][dk][dv], n [H][dk], m [H].
//
// Two forms.
// Steps of few tokens per sequence: mm_step_kernel.  A block owns 64 value columns of one (sequence, head); a lane owns
// four neighbouring columns of every sixteenth row, so the state streams in and out 16 bytes a lane.  Every block forms
// gates and n . q for itself; the block of a (sequence, head) that finishes last writes n and m (when all others have
// read them), and norms the head's result.
// Prompts: chunks of 64 tokens as float32 matrix products.  With F_t the sum of the chunk's f up to t, m_in, S_in, n_in
// the values at its start and n its number of tokens:
//   m_t = F_t + max(m_in, max over s <= t of (i_s - F_s))
//   A_ts = (q_t . k_s) exp(F_t - F_s + i_s - m_t) for s <= t;   c_t = exp(F_t + m_in - m_t)
//   o_t = (sum_s A_ts v_s + c_t S_in^T q_t) / (max(|sum_s A_ts + c_t n_in . q_t|, exp(-m_t)) + 1e-6)
//   S_out = c_n S_in + sum_s exp(F_n - F_s + i_s - m_n) k_s v_s^T,  n_out likewise
// All exponents are at most zero.  F is double: a head that forgets fast reaches sums of several hundred within a chunk,
// and the difference of two of them is the logarithm of a weight.  Kernels: mm_gates (a block per (sequence, head), a wavefront per chunk: prefix sums
// and prefix maxima over the 64 lanes, then m from chunk to chunk), mm_state (each chunk's own share of S and n), mm_carry (the chunks' start
// states in order), mm_out, then the norm.  Matrix instruction layouts as for lightning attention (recurrent.hip).
#include "chunk_form.h"

#define MM_MAX_DK 256
#define MM_VT 128            // value columns per block of the chunk kernels
#define MM_LDS_LIMIT (160 * 1024)

struct MmGates {
  float log_i, log_f;
};
__device__ __forceinline__ MmGates mm_gates(float zi, float zf, float cap, float inv_cap) {
  MmGates g;
  g.log_i = cap * tanhf(zi * inv_cap);
  g.log_f = -blm_softplus(-cap * tanhf(zf * inv_cap));
  return g;
}
__device__ __forceinline__ void mm_store(float* p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ float mm_load(const float* p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }

// ---- few tokens per sequence ----------------------------------------------------------------------
// proj [T][ld] (queries at column 0, keys at H*dk, values at 2*H*dk, output-gate logits at 2*H*dk + H*dv); z [T][ldz]
// float: input-gate logits at column 0, forget-gate logits at H, before their biases.  o_raw [T][H*dv] float.
#define MM_COLS 64
#define MM_ROWS 8           // rows of a lane whose loads are under way together
template <typename TP, typename TA, bool VEC>
__global__ void __launch_bounds__(256)
    mm_step_kernel(const TP* __restrict__ proj, int ld, const float* __restrict__ z, int ldz, const float* __restrict__ bias_i,
                   const float* __restrict__ bias_f, float cap, float q_scale, const float* __restrict__ norm_w, float eps,
                   float* __restrict__ S, float* __restrict__ n_state, float* __restrict__ m_state, float* o_raw,
                   TA* __restrict__ out, const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slots, int T, int B,
                   int H, int dk, int dv, int* arrivals) {
  __shared__ float q_sm[MM_MAX_DK], k_sm[MM_MAX_DK], n_sm[MM_MAX_DK], o_sm[4][MM_COLS], red[32];
  __shared__ int is_last;
  const int ct = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int tid = threadIdx.x, wave = tid / BLM_WAVE, lane = tid & (BLM_WAVE - 1);
  if (b == 0 && ct == 0) {      // padding tokens stand behind the sequences': their rows become zero
    for (int t = cu_seqlens[B]; t < T; ++t)
      for (int j = tid; j < dv; j += 256) out[((size_t)t * H + h) * dv + j] = from_float<TA>(0.f);
  }
  const int slot = seq_slots[b], t0 = cu_seqlens[b], t1 = cu_seqlens[b + 1];
  if (slot < 0 || t1 <= t0) return;      // the same for all blocks of the sequence: none of them is counted
  const int rg = wave * 4 + (lane >> 4), col = ct * MM_COLS + (lane & 15) * 4;
  float* Sh = S + ((size_t)slot * H + h) * dk * dv;
  float* nh = n_state + ((size_t)slot * H + h) * dk;
  float m = m_state[(size_t)slot * H + h];
  for (int i = tid; i < dk; i += 256) n_sm[i] = nh[i];
  const float bi = bias_i[h], bf = bias_f[h], inv_cap = 1.0f / cap;
  float s[MM_ROWS][4];
  auto load_rows = [&](int r0) {
#pragma unroll
    for (int u = 0; u < MM_ROWS; ++u) {
      const int r = r0 + 16 * u;
      if (VEC) {
        const float4 x = (r < dk && col < dv) ? *reinterpret_cast<const float4*>(Sh + (size_t)r * dv + col) : make_float4(0.f, 0.f, 0.f, 0.f);
        s[u][0] = x.x; s[u][1] = x.y; s[u][2] = x.z; s[u][3] = x.w;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) s[u][e] = (r < dk && col + e < dv) ? Sh[(size_t)r * dv + col + e] : 0.f;
      }
    }
  };
  for (int t = t0; t < t1; ++t) {
    load_rows(rg);      // the first rows travel while the gates and the denominator are formed
    const TP* row = proj + (size_t)t * ld;
    const MmGates g = mm_gates(z[(size_t)t * ldz + h] + bi, z[(size_t)t * ldz + H + h] + bf, cap, inv_cap);
    const float m_new = fmaxf(g.log_f + m, g.log_i);
    const float keep = expf(g.log_f + m - m_new), take = expf(g.log_i - m_new);
    m = m_new;
    float vv[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) vv[e] = col + e < dv ? to_float(row[(size_t)2 * H * dk + h * dv + col + e]) * take : 0.f;
    float nq = 0.f;
    for (int i = tid; i < dk; i += 256) {
      const float q = to_float(row[h * dk + i]) * q_scale, k = to_float(row[(size_t)(H + h) * dk + i]);
      const float nn = fmaf(keep, n_sm[i], take * k);
      q_sm[i] = q;
      k_sm[i] = k;
      n_sm[i] = nn;
      nq = fmaf(nn, q, nq);
    }
    nq = block_sum<true>(nq, red);      // its barrier also hands q and k over (four wavefronts)
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int r0 = rg; r0 < dk; r0 += 16 * MM_ROWS) {
      if (r0 != rg) load_rows(r0);
#pragma unroll
      for (int u = 0; u < MM_ROWS; ++u) {
        const int r = r0 + 16 * u;
        const float k = r < dk ? k_sm[r] : 0.f, q = r < dk ? q_sm[r] : 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          s[u][e] = fmaf(keep, s[u][e], k * vv[e]);
          o[e] = fmaf(s[u][e], q, o[e]);
        }
        if (r < dk) {
          if (VEC) {
            if (col < dv) *reinterpret_cast<float4*>(Sh + (size_t)r * dv + col) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (col + e < dv) Sh[(size_t)r * dv + col + e] = s[u][e];
          }
        }
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = rows_sum(o[e]);
    if (lane < 16) {
#pragma unroll
      for (int e = 0; e < 4; ++e) o_sm[wave][lane * 4 + e] = o[e];
    }
    __syncthreads();
    if (tid < MM_COLS && ct * MM_COLS + tid < dv) {
      const float inv = 1.0f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
      mm_store(o_raw + ((size_t)t * H + h) * dv + ct * MM_COLS + tid, (o_sm[0][tid] + o_sm[1][tid] + o_sm[2][tid] + o_sm[3][tid]) * inv);
    }
    // the next token's q, k and o go to the same places: behind everybody's reads of this one's
    if (t + 1 < t1) __syncthreads();
  }
  // stores of results have been acknowledged before this block is counted
  __builtin_amdgcn_s_waitcnt(0x0F70);
  __syncthreads();
  if (tid == 0) {
    const int at = b * H + h;
    const int before = __hip_atomic_fetch_add(arrivals + at, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    is_last = before == (int)gridDim.x - 1;
    if (is_last) __hip_atomic_store(arrivals + at, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (!is_last) return;
  for (int i = tid; i < dk; i += 256) nh[i] = n_sm[i];
  if (tid == 0) m_state[(size_t)slot * H + h] = m;
  for (int t = t0 + wave; t < t1; t += 4) {      // a wavefront per token
    const float* src = o_raw + ((size_t)t * H + h) * dv;
    const TP* grow = proj + (size_t)t * ld + (size_t)2 * H * dk + (size_t)H * dv + (size_t)h * dv;
    float ss = 0.f;
    for (int j = lane; j < dv; j += BLM_WAVE) { const float x = mm_load(src + j); ss = fmaf(x, x, ss); }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)dv + eps);
    for (int j = lane; j < dv; j += BLM_WAVE)
      out[((size_t)t * H + h) * dv + j] = from_float<TA>(mm_load(src + j) * inv * norm_w[h * dv + j] * blm_sigmoid(to_float(grow[j])));
  }
}

// arrivals: B * H counters that are zero before the call and after it.
extern "C" int blm_mm_step(const void* proj, int proj_dtype, int ld, const float* z, int ldz, const float* bias_i, const float* bias_f,
                           float cap, float q_scale, const float* norm_w, float eps, float* S, float* n_state, float* m_state,
                           float* o_raw, void* out, int out_dtype, const int* cu_seqlens, const int* seq_slots, int T, int B, int H,
                           int dk, int dv, int* arrivals, hipStream_t stream) {
  BLM_REQUIRE(T > 0 && B > 0 && B <= 65535 && H > 0 && H <= 65535 && dv > 0, "mm_step: bad sizes T=%d B=%d H=%d dv=%d", T, B, H, dv);
  BLM_REQUIRE(dk >= 1 && dk <= MM_MAX_DK, "mm_step: %d key channels per head are not supported (up to %d)", dk, MM_MAX_DK);
  BLM_REQUIRE(ld >= 2 * H * dk + 2 * H * dv && ldz >= 2 * H && cap > 0.f, "mm_step: rows of %d or %d are too short, or cap %g", ld, ldz, (double)cap);
  const dim3 grid((unsigned)((dv + MM_COLS - 1) / MM_COLS), (unsigned)H, (unsigned)B), block(256);
  const bool vec = dv % 4 == 0 && ((uintptr_t)S & 15) == 0;
#define MM_STEP(TP, TA, V)                                                                                                      \
  hipLaunchKernelGGL((mm_step_kernel<TP, TA, V>), grid, block, 0, stream, (const TP*)proj, ld, z, ldz, bias_i, bias_f, cap, q_scale, \
                     norm_w, eps, S, n_state, m_state, o_raw, (TA*)out, cu_seqlens, seq_slots, T, B, H, dk, dv, arrivals)
#define MM_STEP2(TP, TA) do { if (vec) MM_STEP(TP, TA, true); else MM_STEP(TP, TA, false); } while (0)
  if (proj_dtype == BLM_F32 && out_dtype == BLM_F32) MM_STEP2(float, float);
  else if (proj_dtype == BLM_F32 && out_dtype == BLM_BF16) MM_STEP2(float, bf16);
  else if (proj_dtype == BLM_BF16 && out_dtype == BLM_BF16) MM_STEP2(bf16, bf16);
  else return blm_fail("mm_step: unsupported dtypes %d, %d", proj_dtype, out_dtype);
#undef MM_STEP2
#undef MM_STEP
  BLM_LAUNCH_CHECK("mm_step");
  return 0;
}

// ---- prompts ------------------------------------------------------------------------------------------
// sums [H][T] double: F (the chunk's running sum of log f); gates [2][H][T] float: log i, m; chunk [B][n_seg][H][2] float: m at the chunk's
// start, and c_n, what the chunk leaves of its start state.  Leaves the sequence's m.
#define MM_GATE_WAVES 16
__global__ void __launch_bounds__(MM_GATE_WAVES* BLM_WAVE)
    mm_gates_kernel(const float* __restrict__ z, int ldz, const float* __restrict__ bias_i, const float* __restrict__ bias_f,
                    float cap, double* __restrict__ sums, float* __restrict__ gates, float* __restrict__ chunk,
                    float* __restrict__ m_state,
                    const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slots, int T, int H, int n_seg) {
  __shared__ double F_end[MM_GATE_WAVES], top_end[MM_GATE_WAVES];
  __shared__ float m_at[MM_GATE_WAVES + 1];      // m at the start of each wavefront's chunk, and behind the last one
  const int h = blockIdx.x, b = blockIdx.y, wave = threadIdx.x / BLM_WAVE, lane = threadIdx.x & (BLM_WAVE - 1);
  const int slot = seq_slots[b], first = cu_seqlens[b], n_new = cu_seqlens[b + 1] - first;
  if (slot < 0 || n_new <= 0) return;
  if (threadIdx.x == 0) m_at[MM_GATE_WAVES] = m_state[(size_t)slot * H + h];
  const float bi = bias_i[h], bf = bias_f[h], inv_cap = 1.0f / cap;
  for (int base = 0; base < n_new; base += MM_GATE_WAVES * LC_CHUNK) {      // sixteen chunks at a time
    const int t0 = base + wave * LC_CHUNK, t = t0 + lane;
    const bool valid = t < n_new;
    const float* row = z + (size_t)(first + min(t, n_new - 1)) * ldz;
    const MmGates g = mm_gates(row[h] + bi, row[H + h] + bf, cap, inv_cap);
    double F = valid ? (double)g.log_f : 0.0;
#pragma unroll
    for (int d = 1; d < BLM_WAVE; d <<= 1) {
      const double o = __shfl_up(F, d, BLM_WAVE);
      if (lane >= d) F += o;
    }
    double top = valid ? (double)g.log_i - F : -1e300;
#pragma unroll
    for (int d = 1; d < BLM_WAVE; d <<= 1) {
      const double o = __shfl_up(top, d, BLM_WAVE);
      if (lane >= d) top = fmax(top, o);
    }
    // lanes behind the sequence add nothing to either: the last lane holds the chunk's sum and maximum
    if (lane == BLM_WAVE - 1) { F_end[wave] = F; top_end[wave] = top; }
    __syncthreads();
    if (threadIdx.x == 0) {
      float m = m_at[MM_GATE_WAVES];
      for (int w = 0; w < MM_GATE_WAVES; ++w) {
        m_at[w] = m;
        if (base + w * LC_CHUNK < n_new) m = (float)(F_end[w] + fmax((double)m, top_end[w]));
      }
      m_at[MM_GATE_WAVES] = m;
    }
    __syncthreads();
    if (t0 < n_new) {
      const float m_in = m_at[wave];
      const float m = (float)(F + fmax((double)m_in, top));
      if (valid) {
        const size_t at = (size_t)h * T + first + t;
        sums[at] = F;
        gates[at] = g.log_i;
        gates[(size_t)H * T + at] = m;
      }
      if (lane == BLM_WAVE - 1) {      // its F and m are the chunk's last token's
        float* ck = chunk + (((size_t)b * n_seg + t0 / LC_CHUNK) * H + h) * 2;
        ck[0] = m_in;
        ck[1] = expf((float)(F + (double)m_in - (double)m));
      }
    }
    __syncthreads();      // the next sixteen chunks write the same places
  }
  if (threadIdx.x == 0) m_state[(size_t)slot * H + h] = m_at[MM_GATE_WAVES];
}

// seg_end [B][n_seg][H][dk][dv], seg_n [B][n_seg][H][dk]: what the chunk's own tokens add to S and n by the chunk's end
template <typename TA>
__global__ void __launch_bounds__(LC_THREADS)
    mm_state_kernel(const TA* __restrict__ proj, int ld, const double* __restrict__ sums, const float* __restrict__ gates,
                    float* __restrict__ seg_end,
                    float* __restrict__ seg_n, const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slots, int T, int H,
                    int dk, int dv, int n_seg, int n_vt) {
  extern __shared__ __attribute__((aligned(16))) unsigned char mm_sm[];
  const int c = blockIdx.x, h = blockIdx.y / n_vt, vt = blockIdx.y - h * n_vt, b = blockIdx.z;
  const int slot = seq_slots[b], first = cu_seqlens[b], n_new = cu_seqlens[b + 1] - first;
  const int t0 = c * LC_CHUNK;
  if (slot < 0 || t0 >= n_new) return;
  const int n = min(LC_CHUNK, n_new - t0);
  const int v0 = vt * MM_VT, dvt = min(MM_VT, dv - v0);
  const int DKP = (dk + 31) & ~31, DVP = (dvt + 31) & ~31;
  float* wj = reinterpret_cast<float*>(mm_sm);                      // [64]: the tokens' weights, zero from n on
  TA* Ks = reinterpret_cast<TA*>(wj + LC_CHUNK);                    // [64][DKP]
  TA* Vs = Ks + LC_CHUNK * DKP;                                     // [64][DVP]
  {
    LcOperands<TA, 2> op;
    op.col0[0] = (H + h) * dk; op.width[0] = dk; op.WP[0] = DKP; op.row_ld[0] = DKP; op.dst[0] = Ks;
    op.col0[1] = 2 * H * dk + h * dv + v0; op.width[1] = dvt; op.WP[1] = DVP; op.row_ld[1] = DVP; op.dst[1] = Vs;
    lc_stage<TA, 2>(proj + (size_t)(first + t0) * ld, ld, n, op);
  }
  if (threadIdx.x < LC_CHUNK) {
    const double* F = sums + (size_t)h * T + first + t0;
    const float* I = gates + (size_t)h * T + first + t0;
    const float* M = I + (size_t)H * T;
    const int j = threadIdx.x;
    wj[j] = j < n ? expf((float)(F[n - 1] - F[j] + (double)(I[j] - M[n - 1]))) : 0.f;
  }
  __syncthreads();
  const size_t chunk_at = ((size_t)b * n_seg + c) * H + h;
  if (vt == 0) {
    for (int i = threadIdx.x; i < dk; i += LC_THREADS) {
      float a = 0.f;
      for (int j = 0; j < n; ++j) a = fmaf(wj[j], to_float(Ks[j * DKP + i]), a);
      seg_n[chunk_at * dk + i] = a;
    }
  }
  const int wave = threadIdx.x / BLM_WAVE, lane = threadIdx.x & (BLM_WAVE - 1);
  const int lr = lane & 31, lk = lane >> 5;
  const int NV = DVP / 32, tiles = (DKP / 32) * NV;
  const int depth = (n + 2 * LC_STEPS - 1) & ~(2 * LC_STEPS - 1);
  // sixteen tiles at a time, four per wavefront; a wavefront with fewer repeats the last one into accumulators that are
  // never stored, and the depth is rounded up to what is written out per turn (zeros lie behind the chunk's tokens): no
  // matrix instruction stands under a condition
  for (int tb = 0; tb < tiles; tb += 16) {
    lc_acc acc[4];
    int k_at[4], v_at[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[s][r] = 0.f;
      const int t = min(tb + wave + 4 * s, tiles - 1), tr = t / NV;
      k_at[s] = tr * 32 + lr;
      v_at[s] = (t - tr * NV) * 32 + lr;
    }
    for (int kb = 0; kb < depth; kb += 2 * LC_STEPS) {
#pragma unroll
      for (int u = 0; u < LC_STEPS; ++u) {
        const int k0 = kb + 2 * u;
        const TA* krow = Ks + (k0 + lk) * DKP;
        const TA* vrow = Vs + (k0 + lk) * DVP;
        const float w = wj[k0 + lk];
#pragma unroll
        for (int s = 0; s < 4; ++s)
          acc[s] = __builtin_amdgcn_mfma_f32_32x32x2f32(to_float(krow[k_at[s]]), to_float(vrow[v_at[s]]) * w, acc[s], 0, 0, 0);
      }
    }
    const size_t at = chunk_at * (size_t)dk * dv + v0;
    const bool whole = (dk & 31) == 0 && (dvt & 31) == 0;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int t = tb + wave + 4 * s;
      if (t < tiles) {
        const int tr = t / NV, tc = t - tr * NV;
        const int col = tc * 32 + lr, i0 = tr * 32 + 4 * lk;
        float* end_p = seg_end + at + (size_t)i0 * dv + col;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int di = 8 * (r / 4) + (r & 3);
          if (whole || (i0 + di < dk && col < dvt)) end_p[(size_t)di * dv] = acc[s][r];
        }
      }
    }
  }
}

// From chunk to chunk, S and n alike: start[0] is the sequence's, start[c + 1] = c_n start[c] + end[c]; what comes out
// behind the last chunk is the sequence's new one.  Start values overwrite the ends they are read with.
__global__ void mm_carry_kernel(float* __restrict__ seg_end, float* __restrict__ seg_n, const float* __restrict__ chunk,
                                float* __restrict__ S, float* __restrict__ n_state, const int* __restrict__ cu_seqlens,
                                const int* __restrict__ seq_slots, int H, int dk, int dv, int n_seg) {
  const int b = blockIdx.y;
  const int slot = seq_slots[b];
  const int n_new = cu_seqlens[b + 1] - cu_seqlens[b];
  if (slot < 0 || n_new <= 0) return;
  const int ns = (n_new + LC_CHUNK - 1) / LC_CHUNK;
  const size_t per = (size_t)H * dk * dv, per_n = (size_t)H * dk, per_head = (size_t)dk * dv;
  const float* ck = chunk + (size_t)b * n_seg * H * 2;
  for (size_t e = (size_t)blockIdx.x * blockDim.x + threadIdx.x; e < per + per_n; e += (size_t)gridDim.x * blockDim.x) {
    const bool is_n = e >= per;
    const size_t x = is_n ? e - per : e, stride = is_n ? per_n : per;
    const int h = (int)(x / (is_n ? (size_t)dk : per_head));
    float* state = (is_n ? n_state : S) + (size_t)slot * stride + x;
    float* seg = (is_n ? seg_n : seg_end) + (size_t)b * n_seg * stride + x;
    float v = *state;
    for (int c0 = 0; c0 < ns; c0 += 4) {      // four chunks' loads under way at a time
      float end[4], f[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int c = min(c0 + u, ns - 1);
        end[u] = seg[(size_t)c * stride];
        f[u] = ck[((size_t)c * H + h) * 2 + 1];
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (c0 + u < ns) {
          seg[(size_t)(c0 + u) * stride] = v;
          v = fmaf(f[u], v, end[u]);
        }
    }
    *state = v;
  }
}

template <typename TA>
__global__ void __launch_bounds__(LC_THREADS)
    mm_out_kernel(const TA* __restrict__ proj, int ld, const double* __restrict__ sums, const float* __restrict__ gates,
                  const float* __restrict__ chunk, const float* __restrict__ seg_start, const float* __restrict__ seg_n, float q_scale, float* __restrict__ o_raw,
                  const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slots, int T, int H, int dk, int dv, int n_seg,
                  int n_vt) {
  extern __shared__ __attribute__((aligned(16))) unsigned char mm_sm[];
  const int c = blockIdx.x, h = blockIdx.y / n_vt, vt = blockIdx.y - h * n_vt, b = blockIdx.z;
  const int slot = seq_slots[b], first = cu_seqlens[b], n_new = cu_seqlens[b + 1] - first;
  const int t0 = c * LC_CHUNK;
  if (slot < 0 || t0 >= n_new) return;
  const int n = min(LC_CHUNK, n_new - t0);
  const int v0 = vt * MM_VT, dvt = min(MM_VT, dv - v0);
  const int DKP = (dk + 31) & ~31, DVP = (dvt + 31) & ~31;
  const int SK = DKP + lc_row_pad<TA>();
  double* Fs = reinterpret_cast<double*>(mm_sm);                    // [64] F
  float* As = reinterpret_cast<float*>(Fs + LC_CHUNK);              // [64][65]
  float* Is = As + LC_CHUNK * LC_A_LD;                              // [64] log i
  float* Ms = Is + LC_CHUNK;                                        // [64] m
  float* cs = Ms + LC_CHUNK;                                        // [64] c_t, times q_scale
  float* dn = cs + LC_CHUNK;                                        // [64] one over the denominators
  TA* Qs = reinterpret_cast<TA*>(dn + LC_CHUNK);                    // [64][SK]
  TA* Ks = Qs + LC_CHUNK * SK;                                      // [64][SK]
  TA* Vs = Ks + LC_CHUNK * SK;                                      // [64][DVP]
  {
    LcOperands<TA, 3> op;
    op.col0[0] = h * dk; op.width[0] = dk; op.WP[0] = DKP; op.row_ld[0] = SK; op.dst[0] = Qs;
    op.col0[1] = (H + h) * dk; op.width[1] = dk; op.WP[1] = DKP; op.row_ld[1] = SK; op.dst[1] = Ks;
    op.col0[2] = 2 * H * dk + h * dv + v0; op.width[2] = dvt; op.WP[2] = DVP; op.row_ld[2] = DVP; op.dst[2] = Vs;
    lc_stage<TA, 3>(proj + (size_t)(first + t0) * ld, ld, n, op);
  }
  const size_t chunk_at = ((size_t)b * n_seg + c) * H + h;
  if (threadIdx.x < LC_CHUNK) {
    const size_t row = (size_t)h * T + first + t0;
    const int j = threadIdx.x, at = min(j, n - 1);
    const double fv = sums[row + at];
    const float iv = gates[row + at], mv = gates[(size_t)H * T + row + at];
    Fs[j] = fv;
    Is[j] = iv;
    Ms[j] = mv;
    cs[j] = expf((float)(fv + ((double)chunk[chunk_at * 2] - (double)mv))) * q_scale;
  }
  __syncthreads();
  const int wave = threadIdx.x / BLM_WAVE, lane = threadIdx.x & (BLM_WAVE - 1);
  const int lr = lane & 31, lk = lane >> 5;
  // scores of the three tiles at and below the diagonal, times the tokens' weights
  if (wave < 3) {
    const int ti = wave == 0 ? 0 : 1, tj = wave == 2 ? 1 : 0;
    lc_acc sc;
#pragma unroll
    for (int r = 0; r < 16; ++r) sc[r] = 0.f;
    const TA* qrow = Qs + (ti * 32 + lr) * SK + lk;
    const TA* krow = Ks + (tj * 32 + lr) * SK + lk;
    for (int kb = 0; kb < DKP; kb += 2 * LC_STEPS) {
#pragma unroll
      for (int u = 0; u < LC_STEPS; ++u)
        sc = __builtin_amdgcn_mfma_f32_32x32x2f32(to_float(qrow[kb + 2 * u]), to_float(krow[kb + 2 * u]), sc, 0, 0, 0);
    }
    const int j = tj * 32 + lr;
    const double wj = (double)Is[j] - Fs[j];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int i = ti * 32 + 8 * (r / 4) + 4 * lk + (r & 3);
      As[i * LC_A_LD + j] = (j <= i && i < n) ? sc[r] * q_scale * expf((float)(Fs[i] + wj - (double)Ms[i])) : 0.f;
    }
  } else {
    // the fourth wavefront: n_in . q of every token, times c_t, a lane per token
    const float* ns = seg_n + chunk_at * dk;
    const TA* qrow = Qs + lane * SK;
    float a = 0.f;
    for (int i = 0; i < dk; ++i) a = fmaf(ns[i], to_float(qrow[i]), a);
    dn[lane] = a * cs[lane];
  }
  __syncthreads();
  if (wave == 3) {      // the denominators: a lane per token adds its row of scores
    float a = dn[lane];
    const int top = min(lane, n - 1);
    for (int j = 0; j <= top; ++j) a += As[lane * LC_A_LD + j];
    dn[lane] = 1.0f / (fmaxf(fabsf(a), expf(-Ms[lane])) + 1e-6f);
  }
  const int NV = DVP / 32;
  const int ti = wave & 1, tc0 = wave >> 1;
  const bool two = tc0 + 2 < NV;
  // a wavefront without a first or second tile of its own repeats the last column tile and stores nothing of it
  const int ca = min(tc0, NV - 1) * 32 + lr, cb = min(tc0 + 2, NV - 1) * 32 + lr;
  lc_acc acc[2];
#pragma unroll
  for (int s = 0; s < 2; ++s)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[s][r] = 0.f;
  {   // what the chunk's start state gives
    const float* S0 = seg_start + chunk_at * (size_t)dk * dv + v0;
    const TA* qrow = Qs + (ti * 32 + lr) * SK + lk;
    const float* s0 = S0 + min(ca, dvt - 1);
    const float* s1 = S0 + min(cb, dvt - 1);
    for (int kb = 0; kb < DKP; kb += 2 * LC_STEPS) {
      float sa[LC_STEPS], sb[LC_STEPS];
#pragma unroll
      for (int u = 0; u < LC_STEPS; ++u) {
        const size_t row = (size_t)min(kb + 2 * u + lk, dk - 1) * dv;
        sa[u] = s0[row];
        sb[u] = s1[row];
      }
#pragma unroll
      for (int u = 0; u < LC_STEPS; ++u) {
        const float a = to_float(qrow[kb + 2 * u]);
        acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, sa[u], acc[0], 0, 0, 0);
        acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, sb[u], acc[1], 0, 0, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const float f = cs[ti * 32 + 8 * (r / 4) + 4 * lk + (r & 3)];
      acc[0][r] *= f;
      acc[1][r] *= f;
    }
  }
  {   // what the chunk's own tokens give
    const float* arow = As + (ti * 32 + lr) * LC_A_LD + lk;
    const TA* va = Vs + lk * DVP + ca;
    const TA* vb = Vs + lk * DVP + cb;
    const int depth = min((ti + 1) * 32, (n + 2 * LC_STEPS - 1) & ~(2 * LC_STEPS - 1));
    for (int kb = 0; kb < depth; kb += 2 * LC_STEPS) {
#pragma unroll
      for (int u = 0; u < LC_STEPS; ++u) {
        const int k0 = kb + 2 * u;
        const float a = arow[k0];
        acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, to_float(va[k0 * DVP]), acc[0], 0, 0, 0);
        acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(a, to_float(vb[k0 * DVP]), acc[1], 0, 0, 0);
      }
    }
  }
  __syncthreads();      // the denominators are there
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const int col = (tc0 + 2 * s) * 32 + lr;
    if ((s == 0 ? tc0 < NV : two) && col < dvt) {
      const int i0 = ti * 32 + 4 * lk;
      float* o = o_raw + ((size_t)(first + t0 + i0) * H + h) * dv + v0 + col;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int di = 8 * (r / 4) + (r & 3);
        if (i0 + di < n) o[(size_t)di * H * dv] = acc[s][r] * dn[i0 + di];
      }
    }
  }
}

static size_t mm_state_lds(int dk, int dv, int dtype) {
  const int DKP = (dk + 31) & ~31, DVP = ((dv < MM_VT ? dv : MM_VT) + 31) & ~31;
  return (size_t)LC_CHUNK * sizeof(float) + (size_t)LC_CHUNK * (DKP + DVP) * (dtype == BLM_F32 ? 4 : 2);
}
static size_t mm_out_lds(int dk, int dv, int dtype) {
  const int DKP = (dk + 31) & ~31, DVP = ((dv < MM_VT ? dv : MM_VT) + 31) & ~31;
  const int es = dtype == BLM_F32 ? 4 : 2, SK = DKP + (dtype == BLM_F32 ? 1 : 2);
  return (size_t)(LC_CHUNK * LC_A_LD + 6 * LC_CHUNK) * sizeof(float) + (size_t)LC_CHUNK * (2 * SK + DVP) * es;
}

#define MM_DEVICES 64
static bool g_mm_ready[MM_DEVICES];
// Once per device, outside any stream capture: the chunk kernels take more shared memory than a kernel gets without asking.
extern "C" int blm_mm_chunks_init() {
  int dev = -1;
  hipError_t e = hipGetDevice(&dev);
  BLM_REQUIRE(e == hipSuccess && dev >= 0 && dev < MM_DEVICES, "mm_chunks_init: hipGetDevice failed or device %d is beyond %d", dev, MM_DEVICES);
  const void* ks[] = {(const void*)mm_state_kernel<float>, (const void*)mm_state_kernel<bf16>, (const void*)mm_out_kernel<float>,
                      (const void*)mm_out_kernel<bf16>};
  for (const void* k : ks) {
    e = hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, MM_LDS_LIMIT);
    BLM_REQUIRE(e == hipSuccess, "mm_chunks_init: cannot raise the shared memory limit: %s", hipGetErrorString(e));
  }
  g_mm_ready[dev] = true;
  return 0;
}

extern "C" int blm_mm_chunks_supported(int dk, int dv, int dtype) {
  return (dk >= 1 && dk <= MM_MAX_DK && dv >= 1 && mm_state_lds(dk, dv, dtype) <= MM_LDS_LIMIT && mm_out_lds(dk, dv, dtype) <= MM_LDS_LIMIT) ? 1 : 0;
}

// n_seg: chunks of 64 tokens that cover the longest sequence of the step; sums [H][T] double, gates [2][H][T], chunk [B][n_seg][H][2], seg
// [B][n_seg][H][dk][dv], seg_n [B][n_seg][H][dk] float; o_raw [T][H*dv] float; token_seq: rows of padding tokens become zero.
extern "C" int blm_mm_chunks(const void* proj, int dtype, int ld, const float* z, int ldz, const float* bias_i, const float* bias_f,
                             float cap, float q_scale, const float* norm_w, float eps, float* S, float* n_state, float* m_state,
                             double* sums, float* gates, float* chunk, float* seg, float* seg_n, float* o_raw, void* out, const int* cu_seqlens,
                             const int* seq_slots, const int* token_seq, int T, int B, int H, int dk, int dv, int max_new, int n_seg,
                             hipStream_t stream) {
  const int n_vt = (dv + MM_VT - 1) / MM_VT;
  BLM_REQUIRE(T > 0 && B > 0 && B <= 65535 && H > 0 && (long long)H * n_vt <= 65535, "mm_chunks: bad sizes T=%d B=%d H=%d", T, B, H);
  BLM_REQUIRE(dtype == BLM_F32 || dtype == BLM_BF16, "mm_chunks: unsupported dtype %d", dtype);
  BLM_REQUIRE(blm_mm_chunks_supported(dk, dv, dtype), "mm_chunks: heads of %d x %d channels are not supported", dk, dv);
  BLM_REQUIRE(ld >= 2 * H * dk + 2 * H * dv && ldz >= 2 * H && cap > 0.f, "mm_chunks: rows of %d or %d are too short, or cap %g", ld, ldz, (double)cap);
  BLM_REQUIRE(max_new >= 1 && n_seg >= 1 && (long long)n_seg * LC_CHUNK >= max_new, "mm_chunks: %d chunks do not cover %d tokens", n_seg, max_new);
  int dev = -1;
  BLM_REQUIRE(hipGetDevice(&dev) == hipSuccess && dev >= 0 && dev < MM_DEVICES && g_mm_ready[dev],
              "mm_chunks: blm_mm_chunks_init has not run on device %d", dev);
  hipLaunchKernelGGL(mm_gates_kernel, dim3(H, B), dim3(MM_GATE_WAVES * BLM_WAVE), 0, stream, z, ldz, bias_i, bias_f, cap, sums, gates, chunk, m_state,
                     cu_seqlens, seq_slots, T, H, n_seg);
  BLM_LAUNCH_CHECK("mm_gates");
  const dim3 grid((unsigned)n_seg, (unsigned)(H * n_vt), (unsigned)B);
  const size_t lds_a = mm_state_lds(dk, dv, dtype), lds_c = mm_out_lds(dk, dv, dtype);
  if (dtype == BLM_F32)
    hipLaunchKernelGGL(mm_state_kernel<float>, grid, dim3(LC_THREADS), lds_a, stream, (const float*)proj, ld, sums, gates, seg, seg_n,
                       cu_seqlens, seq_slots, T, H, dk, dv, n_seg, n_vt);
  else
    hipLaunchKernelGGL(mm_state_kernel<bf16>, grid, dim3(LC_THREADS), lds_a, stream, (const bf16*)proj, ld, sums, gates, seg, seg_n,
                       cu_seqlens, seq_slots, T, H, dk, dv, n_seg, n_vt);
  BLM_LAUNCH_CHECK("mm_state");
  const size_t per = (size_t)H * dk * (dv + 1);
  const unsigned cb = (unsigned)((per + 255) / 256 < 2048 ? (per + 255) / 256 : 2048);
  hipLaunchKernelGGL(mm_carry_kernel, dim3(cb, B), dim3(256), 0, stream, seg, seg_n, chunk, S, n_state, cu_seqlens, seq_slots, H, dk,
                     dv, n_seg);
  BLM_LAUNCH_CHECK("mm_carry");
  if (dtype == BLM_F32)
    hipLaunchKernelGGL(mm_out_kernel<float>, grid, dim3(LC_THREADS), lds_c, stream, (const float*)proj, ld, sums, gates, chunk, seg, seg_n,
                       q_scale, o_raw, cu_seqlens, seq_slots, T, H, dk, dv, n_seg, n_vt);
  else
    hipLaunchKernelGGL(mm_out_kernel<bf16>, grid, dim3(LC_THREADS), lds_c, stream, (const bf16*)proj, ld, sums, gates, chunk, seg, seg_n,
                       q_scale, o_raw, cu_seqlens, seq_slots, T, H, dk, dv, n_seg, n_vt);
  BLM_LAUNCH_CHECK("mm_out");
  const char* gate = (const char*)proj + (size_t)(2 * H * dk + H * dv) * (dtype == BLM_F32 ? 4 : 2);
  return blm_launch_head_norm(o_raw, norm_w, H, gate, ld, 1, H, out, dtype, (long long)T * H, dv, eps, token_seq, stream);
}
