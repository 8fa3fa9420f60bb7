// What the recurrent mixers that run prompts in chunks of 64 tokens share: the chunk's sizes, the staging of a chunk's
// rows of one head in shared memory, and the norm of the heads' results (defined in recurrent.hip).
#pragma once
#include "common.h"

__device__ __forceinline__ float blm_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float blm_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float blm_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

#define LC_CHUNK 64
#define LC_MAX 128
#define LC_THREADS 256
#define LC_A_LD (LC_CHUNK + 1)
#define LC_STEPS 8      // matrix instructions written out per turn of a loop over depth: 16 steps of depth
#define LC_LDS_LIMIT (128 * 1024)
typedef float lc_acc __attribute__((ext_vector_type(16)));

template <typename TA>
__device__ __forceinline__ int lc_row_pad() { return sizeof(TA) == 4 ? 1 : 2; }      // an odd number of 4-byte words per row

// A chunk's rows of one head into shared memory as they are, for N operands at once (queries, keys, values): operand p
// is `width[p]` channels from column col0[p] on and arrives in dst[p] [64][row_ld[p]]; the tokens from n on and the channels
// from width up to the padded width WP arrive as zeros.  Where rows and widths allow, every lane takes 16 bytes at a
// time, has all its loads of all operands under way before it turns to the first (one trip to memory, not one per
// operand), and leaves them as 4-byte words (row_ld and the 16-byte pieces keep every word aligned).
template <typename TA, int N>
struct LcOperands {
  int col0[N], width[N], WP[N], row_ld[N];
  TA* dst[N];
};

template <typename TA, int N>
__device__ __forceinline__ void lc_stage(const TA* __restrict__ rows, int ld, int n, const LcOperands<TA, N>& op) {
  constexpr int VEC = 16 / sizeof(TA);
  bool wide = ld % VEC == 0 && (reinterpret_cast<uintptr_t>(rows) & 15) == 0;
#pragma unroll
  for (int p = 0; p < N; ++p) wide = wide && op.width[p] % VEC == 0 && op.col0[p] % VEC == 0 && op.width[p] <= LC_MAX;
  if (wide) {
    // up to 64 * 128 / VEC pieces per operand: at most 4 (16-bit rows) or 8 (float rows) per lane
    constexpr int PER = (LC_CHUNK * LC_MAX / VEC + LC_THREADS - 1) / LC_THREADS;
    uint4 raw[N][PER];
    int at[N][PER];
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const int per_row = op.width[p] / VEC, items = LC_CHUNK * per_row;
      const TA* src = rows + op.col0[p];
#pragma unroll
      for (int u = 0; u < PER; ++u) {
        const int e = threadIdx.x + u * LC_THREADS, j = e / per_row, i = (e - j * per_row) * VEC;
        at[p][u] = e < items ? j * op.row_ld[p] + i : -1;
        raw[p][u] = (e < items && j < n) ? *reinterpret_cast<const uint4*>(src + (size_t)j * ld + i) : uint4{0u, 0u, 0u, 0u};
      }
    }
#pragma unroll
    for (int p = 0; p < N; ++p) {
#pragma unroll
      for (int u = 0; u < PER; ++u) {
        if (at[p][u] >= 0) {
          uint32_t* w = reinterpret_cast<uint32_t*>(op.dst[p] + at[p][u]);
          w[0] = raw[p][u].x; w[1] = raw[p][u].y; w[2] = raw[p][u].z; w[3] = raw[p][u].w;
        }
      }
      if (op.WP[p] > op.width[p]) {
        const int extra = op.WP[p] - op.width[p];
        for (int e = threadIdx.x; e < LC_CHUNK * extra; e += LC_THREADS)
          op.dst[p][(e / extra) * op.row_ld[p] + op.width[p] + e % extra] = from_float<TA>(0.f);
      }
    }
  } else {
#pragma unroll
    for (int p = 0; p < N; ++p) {
      const TA* src = rows + op.col0[p];
      for (int e = threadIdx.x; e < LC_CHUNK * op.WP[p]; e += LC_THREADS) {
        const int j = e / op.WP[p], i = e - j * op.WP[p];
        op.dst[p][j * op.row_ld[p] + i] = (j < n && i < op.width[p]) ? src[(size_t)j * ld + i] : from_float<TA>(0.f);
      }
    }
  }
}

// out[t][h][j] = o_raw[t][h][j] / rms over j * norm_w * f(gate[t][h * dv + j]) for items = tokens * H rows of dv lanes;
// gate rows are gate_ld elements apart (gate null: none), gate_mode 1 sigmoid, 2 SiLU; norm_w holds w_heads rows of dv
// weights (1: shared by all heads, H: one row per head); token_seq (or null): rows of tokens of no sequence become zero.
int blm_launch_head_norm(const float* o_raw, const float* norm_w, int w_heads, const void* gate, int gate_ld, int gate_mode, int H,
                         void* out, int dtype, long long items, int dv, float eps, const int* token_seq, hipStream_t stream);
