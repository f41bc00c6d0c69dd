// The delta rule over a matrix memory whose key rows decay each by a gate of its own.  Per head a
// matrix S [dk, dv], zero before a sequence's first token; for a token with rows q, k [dk], v [dv], decays
// a [dk] in (0, 1] and a step s:
//     S <- diag(a) S;    u = s (v - S^T k);    S <- S + k u^T;    o = S^T q
// With pre-activations z (fp32 products), per head h and key channel i:
//     a = exp(-exp(A_log_h) softplus(z_a[h, i] + dt_bias[h, i])),    s = sigmoid(z_b[h])
// H heads share G key/query heads (head h uses h / (H / G)).  Everything here is fp32.  A request's slot
// begins with S of all heads [H, dk, dv].
//
//   chdelta_scan : token by token; a workgroup per (64 value columns, head, sequence), a wave per 64 key
//                  rows, a thread one column of them in registers.  With the state *before* the token,
//                  S^T k = sum_i k_i a_i S_i and o = sum_i q_i a_i S_i + (k . q) u, so both read-outs share one
//                  pass over S.
#include "common.h"

namespace {
struct ChArgs {
  int H, G, dk, dv;
  int ld, q_off, k_off, v_off;      // rows [tokens, ld] fp32: where the heads of q, k, v begin
  int z_ld, a_off;                  // decay pre-activations [tokens, z_ld] fp32: column a_off + h dk + i
  int b_ld, b_off;                  // step pre-activations [tokens, b_ld] fp32: column b_off + h
  int n_slots, slot_stride;
  int chunk_from;                   // runs of at least so many tokens go chunk by chunk
};

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoidf(float z) { return 1.f / (1.f + expf(-z)); }

constexpr int SCAN_STAGE = 8;      // tokens staged in LDS at a time

// Workgroup (64 value columns, head, sequence) of ceil(dk / ROWS) waves.  Lane l of a wave keeps row l's
// numbers of the token; they reach all lanes as scalars.
template <int ROWS>
__global__ __launch_bounds__(256) void chdelta_scan_kernel(const float* __restrict__ rows, const float* __restrict__ z,
                                                           const float* __restrict__ zb,
                                                           const float* __restrict__ neg_a,
                                                           const float* __restrict__ dt_bias,
                                                           const int* __restrict__ cu_q,
                                                           const int* __restrict__ positions,
                                                           const int* __restrict__ slot_ids, float* __restrict__ state,
                                                           float* __restrict__ out, ChArgs a) {
  extern __shared__ float lds[];
  const int dk = a.dk, dv = a.dv, head = blockIdx.y, seq = blockIdx.z;
  const int kh = head / (a.H / a.G);
  const int lane = threadIdx.x % KVF_WAVE, part = threadIdx.x / KVF_WAVE, parts = blockDim.x / KVF_WAVE;
  const int t0 = cu_q[seq], t1 = cu_q[seq + 1];
  if (t1 <= t0 || (a.chunk_from > 0 && t1 - t0 >= a.chunk_from)) return;
  int slot = slot_ids[seq];
  if (slot < 0 || slot >= a.n_slots) slot = -1;
  float* qs = lds;                               // [STAGE][dk]
  float* ks = qs + SCAN_STAGE * dk;              // [STAGE][dk]
  float* as = ks + SCAN_STAGE * dk;              // [STAGE][dk]
  float* vs = as + SCAN_STAGE * dk;              // [STAGE][64]
  float* gs = vs + SCAN_STAGE * KVF_WAVE;        // [STAGE][2]: step, k . q
  float* psum = gs + SCAN_STAGE * 2;             // [2][parts][2][64]
  const int col = blockIdx.x * KVF_WAVE + lane;
  const bool col_ok = col < dv;
  const int row0 = part * ROWS;
  float* S_slot = slot >= 0 ? state + static_cast<size_t>(slot) * a.slot_stride + static_cast<size_t>(head) * dk * dv
                            : nullptr;
  const bool resume = slot >= 0 && positions[t0] > 0;
  float S[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i)
    S[i] = (resume && col_ok && row0 + i < dk) ? S_slot[static_cast<size_t>(row0 + i) * dv + col] : 0.f;
  const float na = neg_a[head];
  const float* db = dt_bias + static_cast<size_t>(head) * dk;
  int turn = 0;
  for (int tb = t0; tb < t1; tb += SCAN_STAGE) {
    const int cnt = min(SCAN_STAGE, t1 - tb);
    __syncthreads();
    for (int i = threadIdx.x; i < cnt * dk; i += blockDim.x) {
      const int t = i / dk, e = i - t * dk;
      const float* row = rows + static_cast<size_t>(tb + t) * a.ld + kh * dk + e;
      qs[i] = row[a.q_off];
      ks[i] = row[a.k_off];
      as[i] = expf(na * softplus(z[static_cast<size_t>(tb + t) * a.z_ld + a.a_off + head * dk + e] + db[e]));
    }
    for (int i = threadIdx.x; i < cnt * KVF_WAVE; i += blockDim.x) {
      const int t = i / KVF_WAVE, c = blockIdx.x * KVF_WAVE + i % KVF_WAVE;
      vs[i] = c < dv ? rows[static_cast<size_t>(tb + t) * a.ld + a.v_off + head * dv + c] : 0.f;
    }
    if (static_cast<int>(threadIdx.x) < cnt)
      gs[2 * threadIdx.x] = sigmoidf(zb[static_cast<size_t>(tb + threadIdx.x) * a.b_ld + a.b_off + head]);
    __syncthreads();
    for (int t = part; t < cnt; t += parts) {
      float d = 0.f;
      for (int e = lane; e < dk; e += KVF_WAVE) d = fmaf(qs[t * dk + e], ks[t * dk + e], d);
      d = wave_sum(d);
      if (lane == 0) gs[2 * t + 1] = d;
    }
    __syncthreads();
    const int my_row = row0 + lane;
    const bool row_ok = lane < ROWS && my_row < dk;
    for (int t = 0; t < cnt; ++t) {
      const float s = gs[2 * t], kq = gs[2 * t + 1], vv = vs[t * KVF_WAVE + lane];
      const float al = row_ok ? as[t * dk + my_row] : 0.f;      // rows past dk: S stays 0
      const float kf = row_ok ? ks[t * dk + my_row] : 0.f;
      const int ai = __float_as_int(al), kl = __float_as_int(kf), ka = __float_as_int(kf * al);
      const int qa = __float_as_int(row_ok ? qs[t * dk + my_row] * al : 0.f);
      float aq = 0.f, ak = 0.f;
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        aq = fmaf(__int_as_float(__builtin_amdgcn_readlane(qa, i)), S[i], aq);
        ak = fmaf(__int_as_float(__builtin_amdgcn_readlane(ka, i)), S[i], ak);
      }
      if (parts > 1) {
        // the waves' shares in wave order; two buffers in turn, so one barrier a token is enough
        float* ps = psum + turn * parts * 2 * KVF_WAVE;
        turn ^= 1;
        ps[(2 * part) * KVF_WAVE + lane] = aq;
        ps[(2 * part + 1) * KVF_WAVE + lane] = ak;
        __syncthreads();
        aq = 0.f;
        ak = 0.f;
        for (int p = 0; p < parts; ++p) {
          aq += ps[(2 * p) * KVF_WAVE + lane];
          ak += ps[(2 * p + 1) * KVF_WAVE + lane];
        }
      }
      const float u = s * (vv - ak);
      if (part == 0 && col_ok)
        out[(static_cast<size_t>(tb + t) * a.H + head) * dv + col] = fmaf(kq, u, aq);
#pragma unroll
      for (int i = 0; i < ROWS; ++i)
        S[i] = fmaf(__int_as_float(__builtin_amdgcn_readlane(ai, i)), S[i],
                    __int_as_float(__builtin_amdgcn_readlane(kl, i)) * u);
    }
  }
  if (S_slot != nullptr && col_ok) {
#pragma unroll
    for (int i = 0; i < ROWS; ++i)
      if (row0 + i < dk) S_slot[static_cast<size_t>(row0 + i) * dv + col] = S[i];
  }
}

bool args_ok(const ChArgs& a) {
  return a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.H <= 65535 && a.dk > 0 && a.dk <= 256 && a.dv > 0 &&
         a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.q_off + a.G * a.dk <= a.ld && a.k_off + a.G * a.dk <= a.ld &&
         a.v_off + a.H * a.dv <= a.ld && a.a_off >= 0 && a.a_off + a.H * a.dk <= a.z_ld && a.b_off >= 0 &&
         a.b_off + a.H <= a.b_ld && static_cast<long>(a.slot_stride) >= static_cast<long>(a.H) * a.dk * a.dv;
}
}  // namespace

#define CHDELTA_ARGS_DECL                                                                                         \
  const float *rows, int ld, int q_off, int k_off, int v_off, const float *z, int z_ld, int a_off,               \
      const float *zb, int b_ld, int b_off, const float *neg_a, const float *dt_bias, const int *positions,      \
      const int *slot_ids, float *state, int n_slots, int slot_stride, float *out, int H, int G, int dk, int dv

// Runs of fewer than chunk_from tokens (0: all runs), token by token.
KVF_EXPORT int kvf_chdelta_scan(CHDELTA_ARGS_DECL, const int* cu_q, int n_seqs, int chunk_from, hipStream_t s) {
  if (n_seqs <= 0) return 0;
  const ChArgs a{H, G, dk, dv, ld, q_off, k_off, v_off, z_ld, a_off, b_ld, b_off, n_slots, slot_stride, chunk_from};
  if (!args_ok(a) || n_seqs > 65535 || chunk_from < 0) return static_cast<int>(hipErrorInvalidValue);
  const int rows_per = dk <= 32 ? 32 : 64, parts = (dk + rows_per - 1) / rows_per;
  const dim3 grid((dv + KVF_WAVE - 1) / KVF_WAVE, H, n_seqs), block(parts * KVF_WAVE);
  const size_t lds = sizeof(float) * (static_cast<size_t>(SCAN_STAGE) * (3 * dk + KVF_WAVE + 2) +
                                      static_cast<size_t>(4) * parts * KVF_WAVE);
#define GO(R)                                                                                                         \
  hipLaunchKernelGGL((chdelta_scan_kernel<R>), grid, block, lds, s, rows, z, zb, neg_a, dt_bias, cu_q, positions, \
                     slot_ids, state, out, a)
  if (rows_per == 32) GO(32);
  else GO(64);
#undef GO
  return kvf_last_error();
}
