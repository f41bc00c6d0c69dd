// State-space layers: a matrix memory per head with ONE decay per head and token, written either by
// plain outer products or by the delta rule, behind a short causal convolution.  Per head a
// matrix S [dk, dv], zero before a sequence's first token; for a token with rows q, k [dk], v [dv],
// a log decay l <= 0 and a step s:
//     S <- e^l S;    u = s v  (plain)   or   u = s (v - S^T k)  (delta);    S <- S + k u^T;    o = S^T q
// plus, if there are such numbers, D v per head on the output.  With pre-activations z (fp32 products):
//     l = -exp(A_log) softplus(z_a + dt_bias);   s = softplus(z_a + dt_bias)  (plain: the step size itself)
//                                                s = sigmoid(z_b)            (delta)
// H heads share G key/query heads (head h uses h / (H / G)).  Everything here is fp32.  A request's
// slot holds S of all heads [H, dk, dv], then the convolution's last taps - 1 inputs [taps - 1, C]
// (the oldest first).
//
//   ssm_conv   : y_t[c] = silu(sum_j w[c, j] x_(t - (taps-1) + j)[c] + bias[c]) over the rows of a
//                run, what lies before the run taken from the slot (zeros before position 0); the
//                first `unit` channels are heads of dk that become vectors of length one,
//                x / sqrt(sum x^2 + 1e-6), the first half of them (q) times a constant.
//   ssm_scan   : token by token; a workgroup per (64 value columns, head, sequence), a wave per 64
//                key rows, a thread one column of them in registers.  With the state *before* the
//                token, o = e^l S^T q + (k . q) u, so both read-outs share one pass over S.
//   long runs  : cut into chunks of CL tokens (b_t: sum of the chunk's log decays up to t).
//     plain:  ssm_local  every chunk's own contribution K^T diag(e^(b_L - b_s) s_s) V
//             ssm_carry  over a run's chunks in order: the state before every chunk
//     delta:  ssm_solve  the chunk's u solve (I + M) u = diag(s) (v - e^b S0^T k), M[t][r] =
//                        s_t e^(b_t - b_r) k_t . k_r for r < t (lower triangular): T = (I + M)^-1 diag(s)
//             ssm_delta  over a run's chunks in order: R = V - diag(e^b) K S, U = T R,
//                        S <- e^(b_L) S + K^T diag(e^(b_L - b)) U; leaves U and the state before every chunk
//     both:   ssm_read   O = ((Q K^T) * decay, r <= t) U + diag(e^b) Q S0 of all chunks side by side
//                        (the plain form's s_r joins the weights)
//   ssm_gate_norm : y silu(z), then x / rms(x) * w over equal parts of the row.
// The matrix products of the chunks: see memory_chunks.h.
#include "memory_chunks.h"

namespace {
struct SsmArgs {
  int H, G, dk, dv;
  int ld, q_off, k_off, v_off;      // rows [tokens, ld] fp32: where the heads of q, k, v begin
  int z_ld, a_off, b_off;           // gate rows [tokens, z_ld] fp32: columns of z_a and z_b
  int n_slots, slot_floats;
  int chunk_from;                   // runs of at least so many tokens go chunk by chunk
};

// log decay and step of one token and head
template <bool DELTA>
__device__ __forceinline__ void token_gates(const float* __restrict__ z, const SsmArgs& a, int head, float neg_a,
                                            float dt_bias, float& log_decay, float& step) {
  const float dt = softplus(z[a.a_off + head] + dt_bias);
  log_decay = neg_a * dt;
  step = DELTA ? sigmoidf(z[a.b_off + head]) : dt;
}

// ---------------------------------------------------------------------------------- convolution
constexpr int CONV_TILE = 16;      // tokens a thread takes; taps - 1 <= CONV_TILE, so only a run's first tile meets the slot

struct ConvArgs {
  int C, ld_in, col0;               // channels, and where their columns lie in the rows
  int unit, dk;                     // the first `unit` channels are heads of dk that are made unit vectors
  float q_scale;                    // on the first half of those
  int n_slots, slot_floats, state_off;
};

// Grid (channel blocks, tiles of a run, sequences).  A block takes whole heads of the unit
// channels (as many as fit into its threads), or 256 of the others.  The block of a run's first
// tile alone reads the slot's old inputs and writes the new ones, each thread those of its channel.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void ssm_conv_kernel(const T* __restrict__ rows, const float* __restrict__ w,
                                                       const float* __restrict__ bias, const int* __restrict__ cu_q,
                                                       const int* __restrict__ positions,
                                                       const int* __restrict__ slot_ids, float* __restrict__ state,
                                                       float* __restrict__ out, ConvArgs a) {
  __shared__ float sq[CONV_TILE][256];
  __shared__ float factor[CONV_TILE][256];   // per (token, head of the block)
  const int seq = blockIdx.z;
  const int run0 = cu_q[seq], run1 = cu_q[seq + 1];
  const int t0 = run0 + blockIdx.y * CONV_TILE;
  if (t0 >= run1) return;
  const int cnt = min(CONV_TILE, run1 - t0);
  const int per_block = a.unit > 0 ? (256 / a.dk) * a.dk : 256;            // unit channels of a block
  const int unit_blocks = a.unit > 0 ? (a.unit + per_block - 1) / per_block : 0;
  const bool is_unit = static_cast<int>(blockIdx.x) < unit_blocks;
  int c, heads_here = 0;
  if (is_unit) {
    const int base = blockIdx.x * per_block;
    heads_here = min(per_block, a.unit - base) / a.dk;
    c = static_cast<int>(threadIdx.x) < heads_here * a.dk ? base + static_cast<int>(threadIdx.x) : -1;
  } else {
    c = a.unit + (blockIdx.x - unit_blocks) * 256 + threadIdx.x;
    if (c >= a.C) c = -1;
  }
  float y[CONV_TILE];
  if (c >= 0) {
    const T* src = rows + a.col0 + c;
    float x[CONV_TILE + TAPS - 1];          // x[TAPS - 1 + i] is token t0 + i
    if (blockIdx.y == 0) {
      int slot = slot_ids[seq];
      if (slot < 0 || slot >= a.n_slots) slot = -1;
      float* st = slot >= 0 && TAPS > 1 ? state + static_cast<size_t>(slot) * a.slot_floats + a.state_off + c : nullptr;
      const bool resume = st != nullptr && positions[run0] > 0;
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j) x[j] = resume ? st[static_cast<size_t>(j) * a.C] : 0.f;
      if (st != nullptr) {
        // the last TAPS - 1 inputs of (old ones, this run): entry j is input number len + j of the old ones and the run
        const int len = run1 - run0;
        float keep[TAPS > 1 ? TAPS - 1 : 1];
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) {
          const int i = len + j;                                  // < TAPS - 1: an old input
          float old = 0.f;
#pragma unroll
          for (int o = 0; o < TAPS - 1; ++o) old = i == o ? x[o] : old;
          keep[j] = i < TAPS - 1 ? old
                                 : Elem<T>::load(src + static_cast<size_t>(run0 + i - (TAPS - 1)) * a.ld_in);
        }
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) st[static_cast<size_t>(j) * a.C] = keep[j];
      }
    } else {
#pragma unroll
      for (int j = 0; j < TAPS - 1; ++j)
        x[j] = Elem<T>::load(src + static_cast<size_t>(t0 - (TAPS - 1) + j) * a.ld_in);
    }
    // (past the run's end its last row is read again and not used, so that no load is predicated)
#pragma unroll
    for (int i = 0; i < CONV_TILE; ++i)
      x[TAPS - 1 + i] = Elem<T>::load(src + static_cast<size_t>(t0 + min(i, cnt - 1)) * a.ld_in);
    float wt[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) wt[j] = w[static_cast<size_t>(c) * TAPS + j];
    const float b = bias ? bias[c] : 0.f;
#pragma unroll
    for (int i = 0; i < CONV_TILE; ++i) {
      float acc = 0.f;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) acc = fmaf(wt[j], x[i + j], acc);
      acc += b;
      y[i] = acc * sigmoidf(acc);
    }
  }
  if (is_unit) {
    // squares through LDS; eight lanes add up one (token, head)
    const int dk = a.dk, sums = cnt * heads_here, lane8 = threadIdx.x % 8;
    if (c >= 0) {
#pragma unroll
      for (int i = 0; i < CONV_TILE; ++i)
        if (i < cnt) sq[i][threadIdx.x] = y[i] * y[i];
    }
    __syncthreads();
    for (int s = threadIdx.x / 8; s < sums; s += 32) {
      const int i = s / heads_here, h = s - i * heads_here;
      float t = 0.f;
      for (int e = lane8; e < dk; e += 8) t += sq[i][h * dk + e];
      t = group_sum<8>(t);
      if (lane8 == 0) factor[i][h] = 1.f / sqrtf(t + 1e-6f);
    }
    __syncthreads();
    if (c >= 0) {
      const int h = threadIdx.x / dk;
      const float scale = c < a.unit / 2 ? a.q_scale : 1.f;
#pragma unroll
      for (int i = 0; i < CONV_TILE; ++i)
        if (i < cnt) y[i] *= factor[i][h] * scale;
    }
  }
  if (c >= 0) {
#pragma unroll
    for (int i = 0; i < CONV_TILE; ++i)
      if (i < cnt) out[static_cast<size_t>(t0 + i) * a.C + c] = y[i];
  }
}

template <typename T, int TAPS>
int conv_go(const void* rows, const float* w, const float* bias, const int* cu_q, const int* positions,
            const int* slot_ids, float* state, float* out, int n_seqs, int longest, ConvArgs a, hipStream_t s) {
  const int per_block = a.unit > 0 ? (256 / a.dk) * a.dk : 256;
  const int unit_blocks = a.unit > 0 ? (a.unit + per_block - 1) / per_block : 0;
  const dim3 grid(unit_blocks + (a.C - a.unit + 255) / 256, (longest + CONV_TILE - 1) / CONV_TILE, n_seqs);
  hipLaunchKernelGGL((ssm_conv_kernel<T, TAPS>), grid, dim3(256), 0, s, static_cast<const T*>(rows), w, bias, cu_q,
                     positions, slot_ids, state, out, a);
  return kvf_last_error();
}

template <typename T>
int conv_launch(int taps, const void* rows, const float* w, const float* bias, const int* cu_q, const int* positions,
                const int* slot_ids, float* state, float* out, int n_seqs, int longest, ConvArgs a, hipStream_t s) {
#define GO(N) \
  case N: return conv_go<T, N>(rows, w, bias, cu_q, positions, slot_ids, state, out, n_seqs, longest, a, s)
  switch (taps) {
    GO(1); GO(2); GO(3); GO(4); GO(5); GO(6); GO(7); GO(8);
    default: return static_cast<int>(hipErrorInvalidValue);
  }
#undef GO
}

// ---------------------------------------------------------------------------------- token by token
constexpr int SCAN_STAGE = 8;      // tokens staged in LDS at a time

// Workgroup (64 value columns, head, sequence) of ceil(dk / ROWS) waves.  Lane l of a wave keeps
// row l's q and k of the token; every row's numbers reach all lanes as scalars.
template <int ROWS, bool DELTA>
__global__ __launch_bounds__(256) void ssm_scan_kernel(const float* __restrict__ rows, const float* __restrict__ z,
                                                       const float* __restrict__ neg_a,
                                                       const float* __restrict__ dt_bias,
                                                       const float* __restrict__ Dskip, const int* __restrict__ cu_q,
                                                       const int* __restrict__ positions,
                                                       const int* __restrict__ slot_ids, float* __restrict__ state,
                                                       float* __restrict__ out, SsmArgs a) {
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
  float* vs = ks + SCAN_STAGE * dk;              // [STAGE][64]
  float* gs = vs + SCAN_STAGE * KVF_WAVE;        // [STAGE][3]: decay, step, k . q
  float* psum = gs + SCAN_STAGE * 3;             // [2][parts][2][64]
  const int col = blockIdx.x * KVF_WAVE + lane;
  const bool col_ok = col < dv;
  const int row0 = part * ROWS;
  float* S_slot = slot >= 0 ? state + static_cast<size_t>(slot) * a.slot_floats + static_cast<size_t>(head) * dk * dv
                            : nullptr;
  const bool resume = slot >= 0 && positions[t0] > 0;
  float S[ROWS];
#pragma unroll
  for (int i = 0; i < ROWS; ++i)
    S[i] = (resume && col_ok && row0 + i < dk) ? S_slot[static_cast<size_t>(row0 + i) * dv + col] : 0.f;
  const float na = neg_a[head], db = dt_bias[head], dskip = Dskip ? Dskip[head] : 0.f;
  int turn = 0;
  for (int tb = t0; tb < t1; tb += SCAN_STAGE) {
    const int cnt = min(SCAN_STAGE, t1 - tb);
    __syncthreads();
    for (int i = threadIdx.x; i < cnt * dk; i += blockDim.x) {
      const int t = i / dk, e = i - t * dk;
      const float* row = rows + static_cast<size_t>(tb + t) * a.ld + kh * dk + e;
      qs[i] = row[a.q_off];
      ks[i] = row[a.k_off];
    }
    for (int i = threadIdx.x; i < cnt * KVF_WAVE; i += blockDim.x) {
      const int t = i / KVF_WAVE, c = blockIdx.x * KVF_WAVE + i % KVF_WAVE;
      vs[i] = c < dv ? rows[static_cast<size_t>(tb + t) * a.ld + a.v_off + head * dv + c] : 0.f;
    }
    if (static_cast<int>(threadIdx.x) < cnt) {
      float ld, st;
      token_gates<DELTA>(z + static_cast<size_t>(tb + threadIdx.x) * a.z_ld, a, head, na, db, ld, st);
      gs[3 * threadIdx.x] = expf(ld);
      gs[3 * threadIdx.x + 1] = st;
    }
    __syncthreads();
    for (int t = part; t < cnt; t += parts) {
      float d = 0.f;
      for (int e = lane; e < dk; e += KVF_WAVE) d = fmaf(qs[t * dk + e], ks[t * dk + e], d);
      d = wave_sum(d);
      if (lane == 0) gs[3 * t + 2] = d;
    }
    __syncthreads();
    const int my_row = row0 + lane;
    const bool row_ok = lane < ROWS && my_row < dk;
    for (int t = 0; t < cnt; ++t) {
      const float g = gs[3 * t], s = gs[3 * t + 1], kq = gs[3 * t + 2], vv = vs[t * KVF_WAVE + lane];
      const int ql = row_ok ? __float_as_int(qs[t * dk + my_row]) : 0;
      const int kl = row_ok ? __float_as_int(ks[t * dk + my_row]) : 0;
      float aq = 0.f, ak = 0.f;
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        aq = fmaf(__int_as_float(__builtin_amdgcn_readlane(ql, i)), S[i], aq);
        if (DELTA) ak = fmaf(__int_as_float(__builtin_amdgcn_readlane(kl, i)), S[i], ak);
      }
      if (parts > 1) {
        // the waves' shares in wave order; two buffers in turn, so one barrier a token is enough
        float* ps = psum + turn * parts * 2 * KVF_WAVE;
        turn ^= 1;
        ps[(2 * part) * KVF_WAVE + lane] = aq;
        if (DELTA) ps[(2 * part + 1) * KVF_WAVE + lane] = ak;
        __syncthreads();
        aq = 0.f;
        ak = 0.f;
        for (int p = 0; p < parts; ++p) {
          aq += ps[(2 * p) * KVF_WAVE + lane];
          if (DELTA) ak += ps[(2 * p + 1) * KVF_WAVE + lane];
        }
      }
      const float u = DELTA ? s * (vv - g * ak) : s * vv;
      if (part == 0 && col_ok)
        out[(static_cast<size_t>(tb + t) * a.H + head) * dv + col] = fmaf(dskip, vv, fmaf(kq, u, g * aq));
#pragma unroll
      for (int i = 0; i < ROWS; ++i)
        S[i] = fmaf(g, S[i], __int_as_float(__builtin_amdgcn_readlane(kl, i)) * u);
    }
  }
  if (S_slot != nullptr && col_ok) {
#pragma unroll
    for (int i = 0; i < ROWS; ++i)
      if (row0 + i < dk) S_slot[static_cast<size_t>(row0 + i) * dv + col] = S[i];
  }
}

// ---------------------------------------------------------------------------------- chunks
// Sum over a wave's lanes up to each lane's own, in 64 bits: the differences of such sums of log decays
// are what the weights are made of, and a sum that has passed a nearly closed gate is far larger
// than the differences behind it.
__device__ __forceinline__ double running_sum(float v) {
  const int lane = threadIdx.x % KVF_WAVE;
  double b = static_cast<double>(v);
#pragma unroll
  for (int o = 1; o < KVF_WAVE; o <<= 1) {
    const double up = __shfl_up(b, o, KVF_WAVE);
    if (lane >= o) b += up;
  }
  return b;
}

// By the first wave, a lane per token of the chunk: bc[t] = sum of the log decays up to t, sw[t] the
// step.  Tokens past the chunk's count add nothing: bc stays at its last value, sw is zero.
template <bool DELTA, int CL>
__device__ __forceinline__ void chunk_gates(const float* __restrict__ z, const SsmArgs& a, int head, float neg_a,
                                            float dt_bias, int tb, int cnt, double* bc, float* sw) {
  const int lane = threadIdx.x;
  float ld = 0.f, st = 0.f;
  if (lane < cnt) token_gates<DELTA>(z + static_cast<size_t>(tb + lane) * a.z_ld, a, head, neg_a, dt_bias, ld, st);
  const double b = running_sum(ld);
  if (lane < CL) {
    bc[lane] = b;
    sw[lane] = st;
  }
}

// chunks: rows (sequence, first token, tokens, 0).  T [chunks, H, CL, CL]: blocks above the diagonal
// are not written.  B [chunks, H, 2, CL]: e^(b_t), then e^(b_L - b_t) (zero past the chunk's tokens).
template <int DKP, int CL, bool VEC>
__global__ __launch_bounds__(256) void ssm_solve_kernel(const float* __restrict__ rows, const float* __restrict__ z,
                                                        const float* __restrict__ neg_a,
                                                        const float* __restrict__ dt_bias,
                                                        const int* __restrict__ chunks, float* __restrict__ T,
                                                        float* __restrict__ B, SsmArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4, RT = CL / 16;
  double* bc = reinterpret_cast<double*>(lds);   // [CL]
  float* sw = lds + 2 * CL;                      // [CL]
  float* Ks = sw + CL;                           // [CL][QLD]
  float* Ls = Ks + CL * QLD;                     // [CL][TLD]
  float* Ts = Ls + CL * TLD;                     // [CL][TLD]
  const int chunk = blockIdx.y, head = blockIdx.x, kh = head / (a.H / a.G);
  const int tb = chunks[4 * chunk + 1], cnt = chunks[4 * chunk + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  StagedRows<DKP, CL, 256, VEC> ks;
  ks.ask(rows, a, a.k_off + kh * a.dk, tb, cnt);
  if (wave == 0) {
    chunk_gates<true, CL>(z, a, head, neg_a[head], dt_bias[head], tb, cnt, bc, sw);
    if (lane < CL) {
      float* Bg = B + (static_cast<size_t>(chunk) * a.H + head) * 2 * CL;
      Bg[lane] = expf(static_cast<float>(bc[lane]));
      Bg[CL + lane] = lane < cnt ? expf(static_cast<float>(bc[CL - 1] - bc[lane])) : 0.f;
    }
  }
  ks.put(Ks, cnt, a.dk);
  __syncthreads();
  for (int tile = wave; tile < RT * RT; tile += 4) {
    const int rt = tile / RT, ct = tile - rt * RT;
    if (ct > rt) continue;
    const f32x4 acc = mma_rows<DKP>(Ks + (16 * rt + l16) * QLD + 4 * lq, Ks + (16 * ct + l16) * QLD + 4 * lq, zero4());
    const int s = 16 * ct + l16;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int t = 16 * rt + 4 * lq + v;
      Ls[t * TLD + s] = s < t && t < cnt ? sw[t] * expf(static_cast<float>(bc[t] - bc[s])) * acc[v] : 0.f;
    }
  }
  __syncthreads();
  // the diagonal blocks' inverses: wave i block i, lane c column c (forward substitution)
  if (wave < RT) {
    const float* L = Ls + (16 * wave) * TLD + 16 * wave;
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == l16 ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < r; ++s) v = fmaf(-L[r * TLD + s], x[s], v);
      x[r] = v;
    }
    if (lq == 0) {
#pragma unroll
      for (int r = 0; r < 16; ++r) Ts[(16 * wave + r) * TLD + 16 * wave + l16] = x[r];
    }
  }
  __syncthreads();
  // T_ij = -T_ii (sum over j <= k < i of L_ik T_kj), one block diagonal after the other
  for (int d = 1; d < RT; ++d) {
    const int i = d + wave, j = wave;
    if (i < RT) {
      f32x4 p = zero4();
      for (int k = j; k < i; ++k) {
        const f32x4 a4 = *reinterpret_cast<const f32x4*>(Ls + (16 * i + l16) * TLD + 16 * k + 4 * lq);
        const float* tb_ = Ts + (16 * k + 4 * lq) * TLD + 16 * j + l16;
#pragma unroll
        for (int e = 0; e < 4; ++e) p = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[e], tb_[e * TLD], p, 0, 0, 0);
      }
      const f32x4 a4 = *reinterpret_cast<const f32x4*>(Ts + (16 * i + l16) * TLD + 16 * i + 4 * lq);
      f32x4 r = zero4();
#pragma unroll
      for (int e = 0; e < 4; ++e) r = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[e], p[e], r, 0, 0, 0);
#pragma unroll
      for (int v = 0; v < 4; ++v) Ts[(16 * i + 4 * lq + v) * TLD + 16 * j + l16] = -r[v];
    }
    __syncthreads();
  }
  float* Tg = T + (static_cast<size_t>(chunk) * a.H + head) * CL * CL;
  for (int i = tid; i < CL * CL; i += 256) {
    const int t = i / CL, s = i - t * CL;
    if (s / 16 <= t / 16) Tg[i] = Ts[t * TLD + s] * sw[s];
  }
}

// runs: rows (sequence, first chunk, chunks).  Workgroup (16 value columns, head, run).  A chunk's K,
// T, V and B are asked for while the chunk before is worked on.  W [chunks, H, dk, dv] receives the
// state before every chunk, U [tokens, H, dv] the chunks' u.
constexpr int DCOLS = 16;
template <int DKP, int CL, bool VEC>
__global__ __launch_bounds__(256) void ssm_delta_kernel(const float* __restrict__ rows, const int* __restrict__ chunks,
                                                        const int* __restrict__ runs,
                                                        const int* __restrict__ positions,
                                                        const int* __restrict__ slot_ids, float* __restrict__ state,
                                                        const float* __restrict__ T, const float* __restrict__ B,
                                                        float* __restrict__ W, float* __restrict__ U, SsmArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4, RT = CL / 16;
  float* eb = lds;                               // [CL] e^(b_t)
  float* wl = eb + CL;                           // [CL] e^(b_L - b_t)
  float* Ks = wl + CL;                           // [CL][QLD]
  float* Tb = Ks + CL * QLD;                     // [CL][TLD]
  float* Vt = Tb + CL * TLD;                     // [DCOLS][TLD]
  float* Rt = Vt + DCOLS * TLD;                  // [DCOLS][TLD]
  float* Ut = Rt + DCOLS * TLD;                  // [DCOLS][TLD] u times wl
  float* St = Ut + DCOLS * TLD;                  // [DCOLS][QLD]
  const int head = blockIdx.y, col0 = blockIdx.x * DCOLS, kh = head / (a.H / a.G);
  const int seq = runs[3 * blockIdx.z], c0 = runs[3 * blockIdx.z + 1], nc = runs[3 * blockIdx.z + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int dk = a.dk, dv = a.dv;
  int slot = slot_ids[seq];
  if (slot < 0 || slot >= a.n_slots) slot = -1;
  float* S_slot = slot >= 0 ? state + static_cast<size_t>(slot) * a.slot_floats + static_cast<size_t>(head) * dk * dv
                            : nullptr;
  const bool resume = slot >= 0 && positions[chunks[4 * c0 + 1]] > 0;
  for (int i = tid; i < DKP * DCOLS; i += 256) {
    const int r = i / DCOLS, cl = i % DCOLS, c = col0 + cl;
    St[cl * QLD + r] = (resume && r < dk && c < dv) ? S_slot[static_cast<size_t>(r) * dv + c] : 0.f;
  }
  const int k_off = a.k_off + kh * dk, v_off = a.v_off + head * dv;
  constexpr int NT = CL * CL / 4 / 256;
  StagedRows<DKP, CL, 256, VEC> ks;
  StagedTurned<CL, DCOLS, 256, TLD> vs;
  f32x4 treg[NT];
  float breg = 0.f;
  auto ask = [&](int ch, int tb, int cnt) {
    ks.ask(rows, a, k_off, tb, cnt);
    const float* Tg = T + (static_cast<size_t>(ch) * a.H + head) * CL * CL;
#pragma unroll
    for (int x = 0; x < NT; ++x) treg[x] = *reinterpret_cast<const f32x4*>(Tg + 4 * (tid + 256 * x));
    vs.ask(rows + static_cast<size_t>(tb) * a.ld + v_off + col0, a.ld, cnt, dv - col0);
    breg = B[(static_cast<size_t>(ch) * a.H + head) * 2 * CL + tid % (2 * CL)];
  };
  int tb = chunks[4 * c0 + 1], cnt = chunks[4 * c0 + 2];
  ask(c0, tb, cnt);
  for (int j = 0; j < nc; ++j) {
    const int ch = c0 + j;
    // the next chunk's place, asked for early
    const int tb_next = j + 1 < nc ? chunks[4 * (ch + 1) + 1] : 0, cnt_next = j + 1 < nc ? chunks[4 * (ch + 1) + 2] : 0;
    __syncthreads();   // the chunk before is done with everything
    ks.put(Ks, cnt, dk);
#pragma unroll
    for (int x = 0; x < NT; ++x)
      *reinterpret_cast<f32x4*>(Tb + (4 * tid / CL + x * (1024 / CL)) * TLD + 4 * tid % CL) = treg[x];
    vs.put(Vt, cnt, dv - col0);
    if (tid < 2 * CL) eb[tid] = breg;            // (wl lies behind eb)
    __syncthreads();
    if (j + 1 < nc) ask(ch + 1, tb_next, cnt_next);
    // R = V - diag(e^b) K S
    if (wave < RT) {
      const f32x4 acc = mma_rows<DKP>(Ks + (16 * wave + l16) * QLD + 4 * lq, St + l16 * QLD + 4 * lq, zero4());
      const int t = 16 * wave + 4 * lq;
      const f32x4 v4 = *reinterpret_cast<const f32x4*>(Vt + l16 * TLD + t);
      const f32x4 e4 = *reinterpret_cast<const f32x4*>(eb + t);
      f32x4 r;
#pragma unroll
      for (int v = 0; v < 4; ++v) r[v] = fmaf(-e4[v], acc[v], v4[v]);
      *reinterpret_cast<f32x4*>(Rt + l16 * TLD + t) = r;
    }
    __syncthreads();
    // U = T R, over the blocks of T up to the diagonal
    if (wave < RT) {
      const int t = 16 * wave + 4 * lq, c = col0 + l16;
      f32x4 a4[RT], b4[RT], u = zero4();
#pragma unroll
      for (int k = 0; k < RT; ++k) {
        a4[k] = *reinterpret_cast<const f32x4*>(Tb + (16 * wave + l16) * TLD + 16 * k + 4 * lq);
        b4[k] = *reinterpret_cast<const f32x4*>(Rt + l16 * TLD + 16 * k + 4 * lq);
      }
#pragma unroll
      for (int k = 0; k < RT; ++k) {
        if (k > wave) break;
#pragma unroll
        for (int e = 0; e < 4; ++e) u = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[k][e], b4[k][e], u, 0, 0, 0);
      }
      *reinterpret_cast<f32x4*>(Ut + l16 * TLD + t) = u * *reinterpret_cast<const f32x4*>(wl + t);
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (t + v < cnt && c < dv) U[(static_cast<size_t>(tb + t + v) * a.H + head) * dv + c] = u[v];
    }
    __syncthreads();
    // S <- e^(b_L) S + K^T diag(e^(b_L - b)) U; the state as it was goes to W
    const float g_last = eb[CL - 1];
    float* Wg = W + (static_cast<size_t>(ch) * a.H + head) * dk * dv;
    f32x4 b4[RT];
#pragma unroll
    for (int k = 0; k < RT; ++k) b4[k] = *reinterpret_cast<const f32x4*>(Ut + l16 * TLD + 16 * k + 4 * lq);
    for (int kt = wave; kt < DKP / 16; kt += 4) {
      f32x4* mine = reinterpret_cast<f32x4*>(St + l16 * QLD + 16 * kt + 4 * lq);
      const float* ka = Ks + (4 * lq) * QLD + 16 * kt + l16;
      float kv[RT][4];
#pragma unroll
      for (int k = 0; k < RT; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) kv[k][e] = ka[(16 * k + e) * QLD];
      const f32x4 old = *mine;
      f32x4 acc = old * g_last;
#pragma unroll
      for (int k = 0; k < RT; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[k][e], b4[k][e], acc, 0, 0, 0);
      const int c = col0 + l16;
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int r = 16 * kt + 4 * lq + v;
        if (r < dk && c < dv) Wg[static_cast<size_t>(r) * dv + c] = old[v];
      }
      *mine = acc;
    }
    tb = tb_next;
    cnt = cnt_next;
  }
  __syncthreads();
  if (S_slot != nullptr) {
    for (int i = tid; i < DKP * DCOLS; i += 256) {
      const int r = i / DCOLS, cl = i % DCOLS, c = col0 + cl;
      if (r < dk && c < dv) S_slot[static_cast<size_t>(r) * dv + c] = St[cl * QLD + r];
    }
  }
}

// The plain form's chunks alone: W [chunks, H, dk, dv] = K^T diag(e^(b_L - b_s) s_s) V, and E [chunks, H] =
// e^(b_L).  Workgroup (64 value columns, head, chunk).
constexpr int VCOLS = 64;
template <int DKP, int CL, bool VEC>
__global__ __launch_bounds__(256) void ssm_local_kernel(const float* __restrict__ rows, const float* __restrict__ z,
                                                        const float* __restrict__ neg_a,
                                                        const float* __restrict__ dt_bias,
                                                        const int* __restrict__ chunks, float* __restrict__ W,
                                                        float* __restrict__ E, SsmArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4;
  double* bc = reinterpret_cast<double*>(lds);   // [CL]
  float* sw = lds + 2 * CL;                      // [CL]
  float* wl = sw + CL;                           // [CL]
  float* Ks = wl + CL;                           // [CL][QLD]
  float* Vt = Ks + CL * QLD;                     // [VCOLS][TLD]
  const int chunk = blockIdx.z, head = blockIdx.y, col0 = blockIdx.x * VCOLS, kh = head / (a.H / a.G);
  const int tb = chunks[4 * chunk + 1], cnt = chunks[4 * chunk + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int dk = a.dk, dv = a.dv;
  StagedRows<DKP, CL, 256, VEC> ks;
  StagedTurned<CL, VCOLS, 256, TLD> vs;
  ks.ask(rows, a, a.k_off + kh * dk, tb, cnt);
  vs.ask(rows + static_cast<size_t>(tb) * a.ld + a.v_off + head * dv + col0, a.ld, cnt, dv - col0);
  if (wave == 0) {
    chunk_gates<false, CL>(z, a, head, neg_a[head], dt_bias[head], tb, cnt, bc, sw);
    if (lane < CL) wl[lane] = sw[lane] * expf(static_cast<float>(bc[CL - 1] - bc[lane]));
    if (lane == 0 && blockIdx.x == 0)
      E[static_cast<size_t>(chunk) * a.H + head] = expf(static_cast<float>(bc[CL - 1]));
  }
  ks.put(Ks, cnt, dk);
  vs.put(Vt, cnt, dv - col0);
  __syncthreads();
  float* Wg = W + (static_cast<size_t>(chunk) * a.H + head) * dk * dv;
  const int col_tiles = min(VCOLS / 16, (dv - col0 + 15) / 16);
  constexpr int RT = CL / 16;
  for (int kt = wave; 16 * kt < dk; kt += 4) {
    // the tile's rows of K^T, weighted, serve all column tiles
    const float* ka = Ks + (4 * lq) * QLD + 16 * kt + l16;
    float kv[RT][4];
#pragma unroll
    for (int k = 0; k < RT; ++k) {
      const f32x4 w4 = *reinterpret_cast<const f32x4*>(wl + 16 * k + 4 * lq);
#pragma unroll
      for (int e = 0; e < 4; ++e) kv[k][e] = ka[(16 * k + e) * QLD] * w4[e];
    }
    for (int ct = 0; ct < col_tiles; ++ct) {
      f32x4 acc = zero4();
      const float* vb = Vt + (16 * ct + l16) * TLD + 4 * lq;
#pragma unroll
      for (int k = 0; k < RT; ++k) {
        const f32x4 b4 = *reinterpret_cast<const f32x4*>(vb + 16 * k);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[k][e], b4[e], acc, 0, 0, 0);
      }
      const int c = col0 + 16 * ct + l16;
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int r = 16 * kt + 4 * lq + v;
        if (r < dk && c < dv) Wg[static_cast<size_t>(r) * dv + c] = acc[v];
      }
    }
  }
}

// A thread per element of a head's S over the run's chunks in order: W[c] becomes the state before
// chunk c, the state after the last one goes to the slot.  Four chunks' loads are asked for ahead.
__global__ __launch_bounds__(256) void ssm_carry_kernel(const int* __restrict__ chunks, const int* __restrict__ runs,
                                                        const int* __restrict__ positions,
                                                        const int* __restrict__ slot_ids, float* __restrict__ state,
                                                        float* __restrict__ W, const float* __restrict__ E,
                                                        SsmArgs a) {
  const int head = blockIdx.y, e = blockIdx.x * blockDim.x + threadIdx.x;
  const int mat = a.dk * a.dv;
  if (e >= mat) return;
  const int seq = runs[3 * blockIdx.z], c0 = runs[3 * blockIdx.z + 1], nc = runs[3 * blockIdx.z + 2];
  int slot = slot_ids[seq];
  if (slot < 0 || slot >= a.n_slots) slot = -1;
  float* S_slot = slot >= 0 ? state + static_cast<size_t>(slot) * a.slot_floats + static_cast<size_t>(head) * mat + e
                            : nullptr;
  float S = (slot >= 0 && positions[chunks[4 * c0 + 1]] > 0) ? *S_slot : 0.f;
  const size_t gs = static_cast<size_t>(a.H) * mat;
  float* g = W + (static_cast<size_t>(c0) * a.H + head) * mat + e;
  const float* d = E + static_cast<size_t>(c0) * a.H + head;
  int c = 0;
  for (; c + 4 <= nc; c += 4, g += 4 * gs, d += 4 * a.H) {
    const float g0 = g[0], g1 = g[gs], g2 = g[2 * gs], g3 = g[3 * gs];
    const float d0 = d[0], d1 = d[a.H], d2 = d[2 * a.H], d3 = d[3 * a.H];
    g[0] = S;
    S = fmaf(d0, S, g0);
    g[gs] = S;
    S = fmaf(d1, S, g1);
    g[2 * gs] = S;
    S = fmaf(d2, S, g2);
    g[3 * gs] = S;
    S = fmaf(d3, S, g3);
  }
  for (; c < nc; ++c, g += gs, d += a.H) {
    const float g0 = g[0];
    g[0] = S;
    S = fmaf(d[0], S, g0);
  }
  if (S_slot != nullptr) *S_slot = S;
}

// Workgroup of eight waves (64 value columns, head, chunk): the chunk's outputs from the state
// before it (W) and its u (U, or for the plain form v itself with the steps among the weights).
// Wave w has the chunk's rows 16 (w % RT) .. + 15, whose q it keeps in registers for both products;
// K's place in LDS takes the state's columns once the weights are made.
template <int DKP, int CL, bool DELTA, bool VEC>
__global__ __launch_bounds__(512, DKP <= 128 ? 4 : 2) void ssm_read_kernel(
    const float* __restrict__ rows, const float* __restrict__ z, const float* __restrict__ neg_a,
    const float* __restrict__ dt_bias, const float* __restrict__ Dskip, const int* __restrict__ chunks,
    const float* __restrict__ W, const float* __restrict__ U, float* __restrict__ out, SsmArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4, RT = CL / 16, KS = CL > VCOLS ? CL : VCOLS, SHARES = 8 / RT;
  double* bc = reinterpret_cast<double*>(lds);   // [CL]
  float* sw = lds + 2 * CL;                      // [CL]
  float* eb = sw + CL;                           // [CL]
  float* Ks = eb + CL;                           // [CL][QLD], then the state's columns [VCOLS][QLD]
  float* As = Ks + KS * QLD;                     // [CL][TLD]
  float* Ut = As + CL * TLD;                     // [VCOLS][TLD]
  const int chunk = blockIdx.z, head = blockIdx.y, col0 = blockIdx.x * VCOLS, kh = head / (a.H / a.G);
  const int tb = chunks[4 * chunk + 1], cnt = chunks[4 * chunk + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int dk = a.dk, dv = a.dv, rt = wave % RT, share = wave / RT;
  StagedRows<DKP, CL, 512, VEC> ks;
  StagedTurned<CL, VCOLS, 512, TLD> us;
  StagedTurned<DKP, VCOLS, 512, QLD> ws;
  ks.ask(rows, a, a.k_off + kh * dk, tb, cnt);
  f32x4 q4[DKP / 16];
  const bool q_ok = 16 * rt + l16 < cnt;
  {
    const float* p = rows + static_cast<size_t>(tb + 16 * rt + l16) * a.ld + a.q_off + kh * dk;
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) q4[u] = load_four<VEC>(rows, p, 16 * u + 4 * lq, dk, q_ok);
  }
  if (DELTA) us.ask(U + (static_cast<size_t>(tb) * a.H + head) * dv + col0, static_cast<size_t>(a.H) * dv, cnt, dv - col0);
  else us.ask(rows + static_cast<size_t>(tb) * a.ld + a.v_off + head * dv + col0, a.ld, cnt, dv - col0);
  ws.ask(W + (static_cast<size_t>(chunk) * a.H + head) * dk * dv + col0, dv, dk, dv - col0);
  if (wave == 0) {
    chunk_gates<DELTA, CL>(z, a, head, neg_a[head], dt_bias[head], tb, cnt, bc, sw);
    if (lane < CL) eb[lane] = expf(static_cast<float>(bc[lane]));
  }
  ks.put(Ks, cnt, dk);
  us.put(Ut, cnt, dv - col0);
#pragma unroll
  for (int u = 0; u < DKP / 16; ++u) q4[u] = clear_past(q4[u], 16 * u + 4 * lq, dk, q_ok);
  __syncthreads();
  for (int ct = share; ct <= rt; ct += SHARES) {
    f32x4 acc = zero4();
    const float* kb = Ks + (16 * ct + l16) * QLD + 4 * lq;
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) {
      const f32x4 b4 = *reinterpret_cast<const f32x4*>(kb + 16 * u);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[u][e], b4[e], acc, 0, 0, 0);
    }
    const int s = 16 * ct + l16;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int t = 16 * rt + 4 * lq + v;
      float w = 0.f;
      if (s <= t && t < cnt) {
        w = acc[v] * expf(static_cast<float>(bc[t] - bc[s]));
        if (!DELTA) w *= sw[s];
      }
      As[t * TLD + s] = w;
    }
  }
  __syncthreads();   // K is read; its place takes the state
  ws.put(Ks, dk, dv - col0);
  __syncthreads();
  const float dskip = Dskip ? Dskip[head] : 0.f;
  const int col_tiles = min(VCOLS / 16, (dv - col0 + 15) / 16), t4 = 16 * rt + 4 * lq;
  const f32x4 e4 = *reinterpret_cast<const f32x4*>(eb + t4);
  for (int ct = share; ct < col_tiles; ct += SHARES) {
    f32x4 acc = zero4();
    const float* sb = Ks + (16 * ct + l16) * QLD + 4 * lq;
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) {
      const f32x4 b4 = *reinterpret_cast<const f32x4*>(sb + 16 * u);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[u][e], b4[e], acc, 0, 0, 0);
    }
    acc = mma_rows(As + (16 * rt + l16) * TLD + 4 * lq, Ut + (16 * ct + l16) * TLD + 4 * lq, 16 * (rt + 1), acc * e4);
    const int c = col0 + 16 * ct + l16;
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int t = t4 + v;
      if (t >= cnt || c >= dv) continue;
      float o = acc[v];
      if (!DELTA) o = fmaf(dskip, Ut[(16 * ct + l16) * TLD + t], o);
      out[(static_cast<size_t>(tb + t) * a.H + head) * dv + c] = o;
    }
  }
}

template <int DKP, int CL> constexpr size_t solve_lds() { return 4 * (3 * CL + CL * (DKP + 4) + 2 * CL * (CL + 4)); }
template <int DKP, int CL> constexpr size_t delta_lds() {
  return 4 * (2 * CL + CL * (DKP + 4) + CL * (CL + 4) + 3 * DCOLS * (CL + 4) + DCOLS * (DKP + 4));
}
template <int DKP, int CL> constexpr size_t local_lds() { return 4 * (4 * CL + CL * (DKP + 4) + VCOLS * (CL + 4)); }
template <int DKP, int CL> constexpr size_t read_lds() {
  return 4 * (4 * CL + (CL > VCOLS ? CL : VCOLS) * (DKP + 4) + CL * (CL + 4) + VCOLS * (CL + 4));
}

struct ChunkPtrs {
  const float *rows, *z, *neg_a, *dt_bias, *dskip;
  const int *positions, *slot_ids, *chunks, *runs;
  float *state, *out, *T, *B, *W, *U, *E;
  int n_chunks, n_runs;
};

template <int DKP, int CL, bool VEC>
int chunks_go(bool delta, const ChunkPtrs& p, SsmArgs a, hipStream_t s) {
  static bool allowed = false;
  constexpr size_t lds_solve = solve_lds<DKP, CL>(), lds_delta = delta_lds<DKP, CL>(), lds_local = local_lds<DKP, CL>(),
                   lds_read = read_lds<DKP, CL>();
  if (!allowed) {
    hipError_t e = allow_lds(&ssm_solve_kernel<DKP, CL, VEC>, lds_solve);
    if (e == hipSuccess) e = allow_lds(&ssm_delta_kernel<DKP, CL, VEC>, lds_delta);
    if (e == hipSuccess) e = allow_lds(&ssm_local_kernel<DKP, CL, VEC>, lds_local);
    if (e == hipSuccess) e = allow_lds(&ssm_read_kernel<DKP, CL, true, VEC>, lds_read);
    if (e == hipSuccess) e = allow_lds(&ssm_read_kernel<DKP, CL, false, VEC>, lds_read);
    if (e != hipSuccess) return static_cast<int>(e);
    allowed = true;
  }
  const dim3 slices((a.dv + VCOLS - 1) / VCOLS, a.H, p.n_chunks);
  if (delta) {
    hipLaunchKernelGGL((ssm_solve_kernel<DKP, CL, VEC>), dim3(a.H, p.n_chunks), dim3(256), lds_solve, s, p.rows, p.z,
                       p.neg_a, p.dt_bias, p.chunks, p.T, p.B, a);
    hipLaunchKernelGGL((ssm_delta_kernel<DKP, CL, VEC>), dim3((a.dv + DCOLS - 1) / DCOLS, a.H, p.n_runs), dim3(256),
                       lds_delta, s, p.rows, p.chunks, p.runs, p.positions, p.slot_ids, p.state, p.T, p.B, p.W, p.U,
                       a);
    hipLaunchKernelGGL((ssm_read_kernel<DKP, CL, true, VEC>), slices, dim3(512), lds_read, s, p.rows, p.z, p.neg_a,
                       p.dt_bias, p.dskip, p.chunks, p.W, p.U, p.out, a);
  } else {
    hipLaunchKernelGGL((ssm_local_kernel<DKP, CL, VEC>), slices, dim3(256), lds_local, s, p.rows, p.z, p.neg_a,
                       p.dt_bias, p.chunks, p.W, p.E, a);
    hipLaunchKernelGGL(ssm_carry_kernel, dim3((a.dk * a.dv + 255) / 256, a.H, p.n_runs), dim3(256), 0, s, p.chunks,
                       p.runs, p.positions, p.slot_ids, p.state, p.W, p.E, a);
    hipLaunchKernelGGL((ssm_read_kernel<DKP, CL, false, VEC>), slices, dim3(512), lds_read, s, p.rows, p.z, p.neg_a,
                       p.dt_bias, p.dskip, p.chunks, p.W, p.U, p.out, a);
  }
  return kvf_last_error();
}

// ---------------------------------------------------------------------------------- gate and norm
// out[t, :] = w * u / sqrt(mean(u^2) + eps), u = y silu(z), the mean over each of `parts` equal parts of
// the row.  Workgroup (token, part), or with fewer threads a part.  A thread takes eight neighbouring
// elements a load where the rows and parts allow it (V = 8), else one.
template <typename T, int V>
__global__ __launch_bounds__(256) void ssm_gate_norm_kernel(const float* __restrict__ y, const T* __restrict__ z,
                                                            int z_ld, const float* __restrict__ w, float eps,
                                                            T* __restrict__ out, int inner, int size) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, c0 = blockIdx.y * size, step = V * blockDim.x;
  const float* yr = y + static_cast<size_t>(t) * inner + c0;
  const T* zr = z + static_cast<size_t>(t) * z_ld + c0;
  T* o = out + static_cast<size_t>(t) * inner + c0;
  auto gated = [&](int i, float (&u)[V]) {
    float g[V];
    if constexpr (V == 8) {
      load8(yr + i, u);
      load8(zr + i, g);
    } else {
      u[0] = yr[i];
      g[0] = Elem<T>::load(zr + i);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] *= g[e] * sigmoidf(g[e]);
  };
  constexpr int N = V == 8 ? 2 : 8;      // what a thread keeps in registers (the rest is formed twice)
  float u[N][V];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < N; ++k) {
    const int i = V * threadIdx.x + step * k;
    if (i >= size) continue;
    gated(i, u[k]);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(u[k][e], u[k][e], ss);
  }
  for (int i = V * threadIdx.x + step * N; i < size; i += step) {
    float v[V];
    gated(i, v);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(v[e], v[e], ss);
  }
  const float r = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(size) + eps);
  auto put = [&](int i, const float (&v)[V]) {
    if constexpr (V == 8) {
      float wv[8];
      load8(w + c0 + i, wv);
#pragma unroll
      for (int e = 0; e < 8; ++e) wv[e] *= v[e] * r;
      if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<float4*>(o + i) = make_float4(wv[0], wv[1], wv[2], wv[3]);
        *reinterpret_cast<float4*>(o + i + 4) = make_float4(wv[4], wv[5], wv[6], wv[7]);
      } else {
        uint32_t p[4];
#pragma unroll
        for (int e = 0; e < 4; ++e)
          p[e] = static_cast<uint32_t>(f32_to_bf16(wv[2 * e])) | (static_cast<uint32_t>(f32_to_bf16(wv[2 * e + 1])) << 16);
        *reinterpret_cast<uint4*>(o + i) = make_uint4(p[0], p[1], p[2], p[3]);
      }
    } else {
      Elem<T>::store(o + i, v[0] * r * w[c0 + i]);
    }
  };
#pragma unroll
  for (int k = 0; k < N; ++k) {
    const int i = V * threadIdx.x + step * k;
    if (i < size) put(i, u[k]);
  }
  for (int i = V * threadIdx.x + step * N; i < size; i += step) {
    float v[V];
    gated(i, v);
    put(i, v);
  }
}

template <typename T>
int gate_norm_launch(const float* y, const void* z, int z_ld, const float* w, float eps, void* out, int n, int inner,
                     int parts, hipStream_t s) {
  const int size = inner / parts;
  const auto on = [](const void* p, size_t bytes) { return reinterpret_cast<uintptr_t>(p) % bytes == 0; };
  const T* zt = static_cast<const T*>(z);
  T* o = static_cast<T*>(out);
  if (size % 8 == 0 && z_ld % 8 == 0 && on(y, 32) && on(z, 8 * sizeof(T)) && on(w, 32) && on(out, 16)) {
    const int need = (size / 8 + KVF_WAVE - 1) / KVF_WAVE * KVF_WAVE;
    hipLaunchKernelGGL((ssm_gate_norm_kernel<T, 8>), dim3(n, parts), dim3(need < 256 ? need : 256), 0, s, y, zt, z_ld, w,
                       eps, o, inner, size);
  } else {
    hipLaunchKernelGGL((ssm_gate_norm_kernel<T, 1>), dim3(n, parts), dim3(256), 0, s, y, zt, z_ld, w, eps, o, inner, size);
  }
  return kvf_last_error();
}

bool args_ok(const SsmArgs& a, bool delta) {
  return a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.H <= 65535 && a.dk > 0 && a.dk <= 256 && a.dv > 0 &&
         a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.q_off + a.G * a.dk <= a.ld && a.k_off + a.G * a.dk <= a.ld &&
         a.v_off + a.H * a.dv <= a.ld && a.a_off >= 0 && a.a_off + a.H <= a.z_ld &&
         (!delta || (a.b_off >= 0 && a.b_off + a.H <= a.z_ld)) &&
         static_cast<long>(a.slot_floats) >= static_cast<long>(a.H) * a.dk * a.dv;
}
}  // namespace

KVF_EXPORT int kvf_ssm_chunk_len(int dk) { return dk <= 128 ? 64 : 32; }

// rows [tokens, ld_in] (dtype 0 = fp32, 1 = bf16), channels in columns col0 .. col0 + C - 1; w [C, taps]
// and bias [C] (or null) fp32; out [tokens, C] fp32.  unit: how many of the first channels are heads of
// dk to be made unit vectors (q heads, then as many k heads).  longest: the longest run's tokens.
KVF_EXPORT int kvf_ssm_conv(int dtype, const void* rows, int ld_in, int col0, int C, int taps, const float* w,
                            const float* bias, int unit, int dk, float q_scale, const int* cu_q, const int* positions,
                            const int* slot_ids, float* state, int n_slots, int slot_floats, int state_off, float* out,
                            int n_seqs, int longest, hipStream_t s) {
  if (n_seqs <= 0 || longest <= 0) return 0;
  const int tiles = (longest + CONV_TILE - 1) / CONV_TILE;
  if (C <= 0 || col0 < 0 || col0 + C > ld_in || unit < 0 || unit > C || (unit > 0 && (dk <= 0 || dk > 256 || unit % (2 * dk))) ||
      state_off < 0 || static_cast<long>(state_off) + static_cast<long>(taps - 1) * C > slot_floats || n_seqs > 65535 ||
      tiles > 65535)
    return static_cast<int>(hipErrorInvalidValue);
  const ConvArgs a{C, ld_in, col0, unit, dk, q_scale, n_slots, slot_floats, state_off};
  if (dtype == 0)
    return conv_launch<float>(taps, rows, w, bias, cu_q, positions, slot_ids, state, out, n_seqs, longest, a, s);
  if (dtype == 1)
    return conv_launch<bf16_t>(taps, rows, w, bias, cu_q, positions, slot_ids, state, out, n_seqs, longest, a, s);
  return static_cast<int>(hipErrorInvalidValue);
}

#define SSM_ARGS_DECL                                                                                               \
  int delta, const float *rows, int ld, int q_off, int k_off, int v_off, const float *z, int z_ld, int a_off,       \
      int b_off, const float *neg_a, const float *dt_bias, const float *dskip, const int *positions,                \
      const int *slot_ids, float *state, int n_slots, int slot_floats, float *out, int H, int G, int dk, int dv

// Runs of fewer than chunk_from tokens (0: all runs), token by token.
KVF_EXPORT int kvf_ssm_scan(SSM_ARGS_DECL, const int* cu_q, int n_seqs, int chunk_from, hipStream_t s) {
  if (n_seqs <= 0) return 0;
  const SsmArgs a{H, G, dk, dv, ld, q_off, k_off, v_off, z_ld, a_off, b_off, n_slots, slot_floats, chunk_from};
  if (!args_ok(a, delta != 0) || n_seqs > 65535 || chunk_from < 0) return static_cast<int>(hipErrorInvalidValue);
  const int rows_per = dk <= 32 ? 32 : 64, parts = (dk + rows_per - 1) / rows_per;
  const dim3 grid((dv + KVF_WAVE - 1) / KVF_WAVE, H, n_seqs), block(parts * KVF_WAVE);
  const size_t lds = sizeof(float) * (static_cast<size_t>(SCAN_STAGE) * (2 * dk + KVF_WAVE + 3) +
                                      static_cast<size_t>(4) * parts * KVF_WAVE);
#define GO(R, D)                                                                                                   \
  hipLaunchKernelGGL((ssm_scan_kernel<R, D>), grid, block, lds, s, rows, z, neg_a, dt_bias, dskip, cu_q, positions, \
                     slot_ids, state, out, a)
  if (rows_per == 32) {
    if (delta) GO(32, true);
    else GO(32, false);
  } else {
    if (delta) GO(64, true);
    else GO(64, false);
  }
#undef GO
  return kvf_last_error();
}

// The runs named in `runs` (sequence, first chunk, chunks), cut into `chunks` (sequence, first token,
// tokens, 0; at most kvf_ssm_chunk_len(dk) tokens each, a run's chunks in order and one after another).
// Scratch: W [n_chunks, H, dk, dv]; for the delta rule T [n_chunks, H, CL, CL], B [n_chunks, H, 2, CL] and
// U [tokens, H, dv]; for the
// plain form E [n_chunks, H].
KVF_EXPORT int kvf_ssm_chunks(SSM_ARGS_DECL, const int* chunks, int n_chunks, const int* runs, int n_runs, float* T,
                              float* B, float* W, float* U, float* E, hipStream_t s) {
  if (n_chunks <= 0 || n_runs <= 0) return 0;
  const SsmArgs a{H, G, dk, dv, ld, q_off, k_off, v_off, z_ld, a_off, b_off, n_slots, slot_floats, 0};
  if (!args_ok(a, delta != 0) || n_chunks > 65535 || n_runs > 65535 || !chunks || !runs || !W ||
      (delta ? (!T || !B || !U) : !E))
    return static_cast<int>(hipErrorInvalidValue);
  const ChunkPtrs p{rows, z, neg_a, dt_bias, dskip, positions, slot_ids, chunks, runs, state, out, T, B, W, U, E,
                    n_chunks, n_runs};
  const bool vec = dk % 4 == 0 && ld % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(rows) % 16 == 0;
#define GO(DKP, CL) return vec ? chunks_go<DKP, CL, true>(delta != 0, p, a, s) : chunks_go<DKP, CL, false>(delta != 0, p, a, s)
  if (dk <= 32) GO(32, 64);
  if (dk <= 64) GO(64, 64);
  if (dk <= 128) GO(128, 64);
  GO(256, 32);
#undef GO
}

KVF_EXPORT int kvf_ssm_gate_norm(int dtype, const float* y, const void* z, int z_ld, const float* w, float eps, void* out,
                                 int n, int inner, int parts, hipStream_t s) {
  if (n <= 0) return 0;
  if (inner <= 0 || parts <= 0 || inner % parts || parts > 65535) return static_cast<int>(hipErrorInvalidValue);
  if (dtype == 0) return gate_norm_launch<float>(y, z, z_ld, w, eps, out, n, inner, parts, s);
  if (dtype == 1) return gate_norm_launch<bf16_t>(y, z, z_ld, w, eps, out, n, inner, parts, s);
  return static_cast<int>(hipErrorInvalidValue);
}
