// Elementwise gated recurrence (minGRU) of the layered models, fp32: every channel c keeps one number,
//   S <- (1 - z) S + z cand,  z = sigmoid(zr),  cand = u >= 0 ? u + 1/2 : sigmoid(u),  out = S silu(g)
// with zr, u and g projections of the current token alone (biases already added). A step's tokens lie in a packed batch;
// the state is one row of channels per cache slot, taken as zeros by a sequence that starts at position 0.
//
//   lgs_mingru        from the projected rows: token by token, or for prompts in chunks of 32 tokens side by side (a
//                     chunk is S -> A S + L with A the product of its 1 - z and L its result from a zero start)
//   lgs_mingru_step   steps of one token per sequence and few sequences: the three projections of a channel and its
//                     step in one launch, a wave per channel
#include "seq_common.h"

namespace lgs {

struct MinGruArgs {
  const float *z, *u, *g;  // row t of channel c at [t * ld + c]
  long ld;
  float* state;            // [slots][n]
  const int *seq_start, *seq_slot, *seq_pos0;
  float* out;              // [T][n]
  uint16_t* out16;         // instead of out
  int n;
  float* ws;               // prompt form: [B * max_chunks][2][n]: A and L, then A and the state at the chunk's start
  int max_chunks;
};

constexpr int kGruChunk = 32, kGruBatch = 8;

// one token: gate and candidate of (zr, u), applied to S; `keep` receives 1 - z
__device__ __forceinline__ float mingru_next(float zr, float u, float S, float& keep) {
  const float e = expf(-fabsf(zr)), q = 1.0f / (1.0f + e), r = e * q;  // sigmoid(|zr|), sigmoid(-|zr|)
  const float gate = zr >= 0.0f ? q : r;
  keep = zr >= 0.0f ? r : q;
  const float cand = u >= 0.0f ? u + 0.5f : sigmoid_f(u);
  return fmaf(keep, S, gate * cand);
}

// grid (ceil(n / 256), chunks, B): thread = channel. MODE 0: the whole sequence from its stored state (grid.y 1); MODE 1:
// a chunk's A and L; MODE 2: a chunk's outputs from its start state. A batch of tokens is fetched before it is walked.
template <int MODE>
__global__ void __launch_bounds__(256) mingru_kernel(MinGruArgs p) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, n = p.n;
  const int r0 = p.seq_start[b], len = p.seq_start[b + 1] - r0;
  const int first = MODE == 0 ? 0 : blockIdx.y * kGruChunk;
  if (c >= n || first >= len) return;
  const int last = MODE == 0 ? len : min(len, first + kGruChunk);
  const size_t slot = p.seq_slot[b];
  float* w = MODE == 0 ? nullptr : p.ws + ((size_t)b * p.max_chunks + blockIdx.y) * 2 * n + c;
  float S = 0.0f, A = 1.0f;
  if (MODE == 0 && p.seq_pos0[b] > 0) S = p.state[slot * n + c];
  if (MODE == 2) S = w[n];
  for (int t0 = first; t0 < last; t0 += kGruBatch) {
    float z[kGruBatch], u[kGruBatch], g[kGruBatch];
#pragma unroll
    for (int t = 0; t < kGruBatch; ++t) {
      const size_t at = (size_t)(r0 + min(t0 + t, last - 1)) * p.ld + c;  // (rows past the end repeat the last, unused)
      z[t] = p.z[at];
      u[t] = p.u[at];
      g[t] = MODE != 1 ? p.g[at] : 0.0f;
    }
#pragma unroll
    for (int t = 0; t < kGruBatch; ++t) {
      if (t0 + t >= last) break;
      float keep;
      S = mingru_next(z[t], u[t], S, keep);
      if (MODE == 1) {
        A *= keep;
      } else {
        const float v = S * (g[t] * sigmoid_f(g[t]));
        const size_t at = (size_t)(r0 + t0 + t) * n + c;
        if (p.out16) p.out16[at] = f2bf(v);
        else p.out[at] = v;
      }
    }
  }
  if (MODE == 0) p.state[slot * n + c] = S;
  if (MODE == 1) w[0] = A, w[n] = S;
}

// grid (ceil(n / 64), B): per channel the recurrence over a sequence's chunks: L becomes the state at the chunk's start,
// and the state after the last chunk goes to the slot
__global__ void __launch_bounds__(64) mingru_carry_kernel(MinGruArgs p) {
  const int c = blockIdx.x * 64 + threadIdx.x, b = blockIdx.y, n = p.n;
  if (c >= n) return;
  const int len = p.seq_start[b + 1] - p.seq_start[b], chunks = (len + kGruChunk - 1) / kGruChunk;
  float* st = p.state + (size_t)p.seq_slot[b] * n + c;
  float* w = p.ws + (size_t)b * p.max_chunks * 2 * n + c;
  float S = p.seq_pos0[b] > 0 ? *st : 0.0f;
  constexpr int U = 16;  // chunks fetched side by side
  for (int k0 = 0; k0 < chunks; k0 += U) {
    float A[U], L[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const float* q = w + (size_t)min(k0 + i, chunks - 1) * 2 * n;
      A[i] = q[0];
      L[i] = q[n];
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (k0 + i >= chunks) break;
      w[(size_t)(k0 + i) * 2 * n + n] = S;
      S = fmaf(A[i], S, L[i]);
    }
  }
  *st = S;
}

struct MinGruStepArgs {
  const float* h;  // [M][ldh] the layer's normed input
  long ldh;
  const void* w;   // [rows][K]; channel c's rows of the three projections at z0 + c, u0 + c, g0 + c
  const float* bias;  // [rows] or null
  int z0, u0, g0, M, K, n;
  float* state;
  const int *seq_slot, *seq_pos0;
  float* out;      // [M][n]
};

// grid (ceil(n / 4)): wave = channel
template <bool WF32, int MT>
__global__ void __launch_bounds__(256) mingru_step_kernel(MinGruStepArgs p) {
  const int lane = threadIdx.x & 63, c = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (c >= p.n) return;
  const int K = p.K;
  const int rows[3] = {p.z0 + c, p.u0 + c, p.g0 + c};
  // lane m finishes row m: its state is fetched ahead of the products
  const bool fin = lane < p.M;
  const size_t at = fin ? (size_t)p.seq_slot[lane] * p.n + c : 0;
  const float S0 = fin && p.seq_pos0[lane] > 0 ? p.state[at] : 0.0f;
  float bias[3];
#pragma unroll
  for (int r = 0; r < 3; ++r) bias[r] = p.bias ? p.bias[rows[r]] : 0.0f;
  float acc[MT][3];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 3; ++r) acc[m][r] = 0.0f;
  if ((K & 7) == 0 && (p.ldh & 3) == 0 && ((uintptr_t)p.h & 15) == 0 && ((uintptr_t)p.w & 15) == 0) {
#pragma unroll 2
    for (int k = lane * 8; k < K; k += 512) {
      float wv[3][8];
#pragma unroll
      for (int r = 0; r < 3; ++r) wload8<WF32>(p.w, (size_t)rows[r] * K + k, wv[r]);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        if (m >= p.M) continue;
        const float* hr = p.h + (size_t)m * p.ldh + k;
        const float4 lo = *(const float4*)hr, hi = *(const float4*)(hr + 4);
        const float hv[8] = {lo.x, lo.y, lo.z, lo.w, hi.x, hi.y, hi.z, hi.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float x = aop<WF32>(hv[e]);
#pragma unroll
          for (int r = 0; r < 3; ++r) acc[m][r] = fmaf(x, wv[r][e], acc[m][r]);
        }
      }
    }
  } else {
    for (int k = lane; k < K; k += 64) {
      float wv[3];
#pragma unroll
      for (int r = 0; r < 3; ++r) wv[r] = wload<WF32>(p.w, (size_t)rows[r] * K + k);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        if (m >= p.M) continue;
        const float x = aop<WF32>(p.h[(size_t)m * p.ldh + k]);
#pragma unroll
        for (int r = 0; r < 3; ++r) acc[m][r] = fmaf(x, wv[r], acc[m][r]);
      }
    }
  }
  float v[3] = {0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 3; ++r) {
      const float s = wave_sum(acc[m][r]);
      if (lane == m) v[r] = s + bias[r];
    }
  if (!fin) return;
  float keep;
  const float S = mingru_next(v[0], v[1], S0, keep);
  p.state[at] = S;
  p.out[(size_t)lane * p.n + c] = S * (v[2] * sigmoid_f(v[2]));
}

}  // namespace lgs

extern "C" int lgs_mingru(const float* z, const float* u, const float* g, long ld, float* state, const int* seq_start,
                          const int* seq_slot, const int* seq_pos0, void* out, int out_bf16, int B, int n, float* ws,
                          int max_chunks, hipStream_t stream) {
  LGA_CHECK_ARG(z && u && g && state && seq_start && seq_slot && seq_pos0 && out, "lgs_mingru: null pointer");
  LGA_CHECK_ARG(B > 0 && B <= 65535 && n > 0 && ld >= n, "lgs_mingru: bad sizes");
  LGA_CHECK_ARG(!ws || (max_chunks > 0 && max_chunks <= 65535), "lgs_mingru: the longest sequence's chunks (up to 65535)");
  lgs::MinGruArgs p{z, u, g, ld, state, seq_start, seq_slot, seq_pos0, out_bf16 ? nullptr : (float*)out,
                    out_bf16 ? (uint16_t*)out : nullptr, n, ws, max_chunks};
  const unsigned cols = (n + 255) / 256;
  if (!ws) {
    lgs::mingru_kernel<0><<<dim3(cols, 1, B), 256, 0, stream>>>(p);
  } else {
    lgs::mingru_kernel<1><<<dim3(cols, max_chunks, B), 256, 0, stream>>>(p);
    lgs::mingru_carry_kernel<<<dim3((n + 63) / 64, B), 64, 0, stream>>>(p);
    lgs::mingru_kernel<2><<<dim3(cols, max_chunks, B), 256, 0, stream>>>(p);
  }
  LGA_LAUNCH_RETURN();
}

extern "C" int lgs_mingru_step(const float* h, long ldh, const void* w, int w_f32, const float* bias, int z0, int u0, int g0,
                               int rows, int M, int K, int n, float* state, const int* seq_slot, const int* seq_pos0,
                               float* out, hipStream_t stream) {
  LGA_CHECK_ARG(h && w && state && seq_slot && seq_pos0 && out, "lgs_mingru_step: null pointer");
  LGA_CHECK_ARG(M > 0 && M <= 8 && K > 0 && n > 0 && ldh >= K, "lgs_mingru_step: 1 to 8 sequences of one token each");
  LGA_CHECK_ARG(z0 >= 0 && u0 >= 0 && g0 >= 0 && (long)z0 + n <= rows && (long)u0 + n <= rows && (long)g0 + n <= rows,
                "lgs_mingru_step: projections outside the matrix");
  lgs::MinGruStepArgs p{h, ldh, w, bias, z0, u0, g0, M, K, n, state, seq_slot, seq_pos0, out};
  const unsigned grid = (n + 3) / 4;
#define LGS_GRU(MT)                                                               \
  do {                                                                            \
    if (w_f32) lgs::mingru_step_kernel<true, MT><<<grid, 256, 0, stream>>>(p);    \
    else lgs::mingru_step_kernel<false, MT><<<grid, 256, 0, stream>>>(p);         \
  } while (0)
  if (M == 1) LGS_GRU(1);
  else if (M == 2) LGS_GRU(2);
  else if (M <= 4) LGS_GRU(4);
  else LGS_GRU(8);
#undef LGS_GRU
  LGA_LAUNCH_RETURN();
}
