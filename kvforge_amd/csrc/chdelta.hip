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
//   long runs    : cut into chunks of CL tokens.  With P(r, t) the product of the decays of the tokens r + 1 .. t
//                  (a number per key channel) the chunk's u solve (I + M) u = diag(s) (v - Kd S0), Kd_t = k_t P(0, t),
//                  M[t][r] = s_t sum_i k_t P(r, t) k_r for r < t; the state behind the chunk is P(0, L) S0 + Kw^T U,
//                  Kw_t = k_t P(t, L); the outputs are A U + Qd S0, A[t][r] = sum_i q_t P(r, t) k_r for r <= t,
//                  Qd_t = q_t P(0, t).
//     chdelta_solve  all chunks side by side: T = (I + M)^-1 diag(s), A, Kd, Kw, Qd, P(0, L)
//     chdelta_delta  over a run's chunks in order: R = V - Kd S, U = T R, S <- P(0, L) S + Kw^T U; leaves U
//                    and the state before every chunk
//     chdelta_read   the outputs, all chunks side by side
// M and A are matrix products of scaled rows, but no single scale per token will do: P(r, t) = x_t / x_r
// with one running product x overflows where a gate is nearly closed.  So the pairs (t, r) are sorted by
// the place where the two tokens' paths part in a binary tree over the chunk: tokens of one block of
// 2 s, t in its upper and r in its lower half, have P(r, t) = (product over the upper half up to t) (product
// over the lower half behind r).  Both factors are products of decays, at most one, and nothing is ever
// divided.  A level of the tree is one 16 x 16 product per block of 16 tokens, of which the level's own
// pairs are kept; blocks of 16 against each other take the blocks' products up to t and behind r, and
// those of the blocks between.
#include "memory_chunks.h"

namespace {
struct ChArgs {
  int H, G, dk, dv;
  int ld, q_off, k_off, v_off;      // rows [tokens, ld] fp32: where the heads of q, k, v begin
  int z_ld, a_off;                  // decay pre-activations [tokens, z_ld] fp32: column a_off + h dk + i
  int b_ld, b_off;                  // step pre-activations [tokens, b_ld] fp32: column b_off + h
  int n_slots, slot_stride;
  int chunk_from;                   // runs of at least so many tokens go chunk by chunk
};

// A key channel's decay exp(-A softplus(z)), neg_a = -A.  With x = e^-|z| and u = 1 + x rounded, log1p(x) =
// log(u) x / (u - 1), which keeps small x whole: a channel that hardly fades has softplus(z) ~ x far below the
// rounding of 1 + x.  (The hardware's exponential and logarithm: within an ulp or so.)
__device__ __forceinline__ float decay_of(float z, float neg_a) {
  const float x = __expf(-fabsf(z)), u = 1.f + x, d = u - 1.f;
  const float l = d == 0.f ? x : __logf(u) * __fdividef(x, d);
  return __expf(neg_a * (fmaxf(z, 0.f) + l));
}

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
      as[i] = decay_of(z[static_cast<size_t>(tb + t) * a.z_ld + a.a_off + head * dk + e] + db[e], na);
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

// ---------------------------------------------------------------------------------- chunks
// A thread per (key channel, block of 16 tokens): it keeps the channel's q, k, decays and products over the
// block in registers, and puts the level's scaled rows down in LDS for all waves.
// chunks: rows (sequence, first token, tokens, 0).  T, A [chunks, H, CL, CL] (blocks above the diagonal are not
// written), E [chunks, H, dk] = P(0, L), Kd, Kw, Qd [tokens, H, dk].
template <int DKP, int CL> constexpr int solve_threads() { return DKP * (CL / 16); }
template <int DKP, int CL> constexpr size_t solve_lds() {
  return 4 * (3 * CL * (DKP + 4) + 2 * CL * (CL + 4) + (CL / 16) * DKP + CL);
}

template <int DKP, int CL>
__global__ __launch_bounds__(DKP * (CL / 16)) void chdelta_solve_kernel(
    const float* __restrict__ rows, const float* __restrict__ z, const float* __restrict__ zb,
    const float* __restrict__ neg_a, const float* __restrict__ dt_bias, const int* __restrict__ chunks,
    float* __restrict__ T, float* __restrict__ A, float* __restrict__ E, float* __restrict__ Kd, float* __restrict__ Kw,
    float* __restrict__ Qd, ChArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int RT = CL / 16, NT = solve_threads<DKP, CL>(), WAVES = NT / KVF_WAVE, QLD = DKP + 4, TLD = CL + 4;
  constexpr int JOBS = 2 * RT > WAVES ? 2 * RT / WAVES : 1;      // blocks of the diagonal a wave works on, for M or for A
  float* Lk = lds;                    // [CL][QLD] k as the left factor
  float* Lq = Lk + CL * QLD;          // [CL][QLD] q likewise
  float* Rk = Lq + CL * QLD;          // [CL][QLD] k as the right factor
  float* Ls = Rk + CL * QLD;          // [CL][TLD] M
  float* Ts = Ls + CL * TLD;          // [CL][TLD]
  float* tot = Ts + CL * TLD;         // [RT][DKP] products over whole blocks
  float* sw = tot + RT * DKP;         // [CL] steps
  const int chunk = blockIdx.y, head = blockIdx.x, kh = head / (a.H / a.G);
  const int tb = chunks[4 * chunk + 1], cnt = chunks[4 * chunk + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int ch = tid % DKP, sub = tid / DKP, dk = a.dk;
  const bool ch_ok = ch < dk;
  const size_t mat = (static_cast<size_t>(chunk) * a.H + head) * CL * CL;
  float q[16], k[16], pre[16], suf[16];
  {
    const int e = ch_ok ? ch : dk - 1;
    const float* qp = rows + a.q_off + kh * dk + e;
    const float* kp = rows + a.k_off + kh * dk + e;
    const float* zp = z + a.a_off + head * dk + e;
    // (past the chunk's tokens its last row is read again, so that no load is predicated)
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const size_t row = tb + min(16 * sub + j, cnt - 1);
      q[j] = qp[row * a.ld];
      k[j] = kp[row * a.ld];
      pre[j] = zp[row * a.z_ld];
    }
    const float na = neg_a[head], db = dt_bias[head * dk + e];
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const bool in = 16 * sub + j < cnt;
      q[j] = in && ch_ok ? q[j] : 0.f;
      k[j] = in && ch_ok ? k[j] : 0.f;
      pre[j] = in ? decay_of(pre[j] + db, na) : 1.f;
      suf[j] = 1.f;
    }
  }
  if (tid < CL) sw[tid] = tid < cnt ? sigmoidf(zb[static_cast<size_t>(tb + tid) * a.b_ld + a.b_off + head]) : 0.f;
  const int at = 16 * sub * QLD + ch;
  // the pairs (t, t) of A: no decay at all
#pragma unroll
  for (int j = 0; j < 16; ++j) {
    Lq[at + j * QLD] = q[j];
    Rk[at + j * QLD] = k[j];
  }
  __syncthreads();
  f32x4 res[JOBS];
#pragma unroll
  for (int x = 0; x < JOBS; ++x) {
    const int job = wave + x * WAVES, b = job % RT;
    res[x] = zero4();
    if (job >= RT && job < 2 * RT) {
      const f32x4 acc = mma_rows<DKP>(Lq + (16 * b + l16) * QLD + 4 * lq, Rk + (16 * b + l16) * QLD + 4 * lq, zero4());
#pragma unroll
      for (int v = 0; v < 4; ++v) res[x][v] = 4 * lq + v == l16 ? acc[v] : 0.f;
    }
  }
  __syncthreads();
#pragma unroll
  for (int s = 1; s <= 16; s *= 2) {
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      Lk[at + j * QLD] = k[j] * pre[j];
      Lq[at + j * QLD] = q[j] * pre[j];
      Rk[at + j * QLD] = k[j] * suf[j];
    }
    if (s == 16) break;        // the blocks' own products are there: what lies between blocks comes below
    __syncthreads();
#pragma unroll
    for (int x = 0; x < JOBS; ++x) {
      const int job = wave + x * WAVES, b = job % RT;
      if (job < 2 * RT) {
        const float* L = job < RT ? Lk : Lq;
        const f32x4 acc = mma_rows<DKP>(L + (16 * b + l16) * QLD + 4 * lq, Rk + (16 * b + l16) * QLD + 4 * lq, zero4());
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          const int t = 4 * lq + v, d = t ^ l16;
          if (t > l16 && d >= s && d < 2 * s) res[x][v] = acc[v];
        }
      }
    }
    // products over blocks of 2 s from those over blocks of s
#pragma unroll
    for (int b = 0; b < 16; b += 2 * s) {
      const float lower = pre[b + s - 1], upper = pre[b + 2 * s - 1];
#pragma unroll
      for (int j = 0; j < s; ++j) {
        pre[b + s + j] *= lower;
        suf[b + j] *= upper;
      }
    }
    __syncthreads();
  }
  tot[sub * DKP + ch] = pre[15];
#pragma unroll
  for (int x = 0; x < JOBS; ++x) {
    const int job = wave + x * WAVES, b = job % RT;
    if (job < 2 * RT) {
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int t = 4 * lq + v;
        if (job < RT) Ls[(16 * b + t) * TLD + 16 * b + l16] = sw[16 * b + t] * res[x][v];
        else A[mat + (16 * b + t) * CL + 16 * b + l16] = res[x][v];
      }
    }
  }
  __syncthreads();
  // blocks of 16 against each other
  for (int job = wave; job < RT * (RT - 1); job += WAVES) {
    const int pair = job >> 1;                       // (1, 0), (2, 0), (2, 1), (3, 0), (3, 1), (3, 2)
    const int i = pair < 1 ? 1 : pair < 3 ? 2 : 3, j = pair - i * (i - 1) / 2;
    const float* L = ((job & 1) ? Lq : Lk) + (16 * i + l16) * QLD + 4 * lq;
    const float* R = Rk + (16 * j + l16) * QLD + 4 * lq;
    f32x4 acc = zero4();
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) {
      const f32x4 a4 = *reinterpret_cast<const f32x4*>(L + 16 * u);
      f32x4 b4 = *reinterpret_cast<const f32x4*>(R + 16 * u);
      for (int m = j + 1; m < i; ++m) b4 *= *reinterpret_cast<const f32x4*>(tot + m * DKP + 16 * u + 4 * lq);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[e], b4[e], acc, 0, 0, 0);
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int t = 16 * i + 4 * lq + v, r = 16 * j + l16;
      if (job & 1) A[mat + t * CL + r] = acc[v];
      else Ls[t * TLD + r] = sw[t] * acc[v];
    }
  }
  if (ch_ok) {
    float before = 1.f, behind = 1.f;
#pragma unroll
    for (int m = 0; m < RT; ++m) {
      before *= m < sub ? tot[m * DKP + ch] : 1.f;
      behind *= m > sub ? tot[m * DKP + ch] : 1.f;
    }
    const size_t step = static_cast<size_t>(a.H) * dk;
    size_t o = static_cast<size_t>(tb + 16 * sub) * step + head * dk + ch;
#pragma unroll
    for (int j = 0; j < 16; ++j, o += step) {
      if (16 * sub + j >= cnt) continue;
      const float x = pre[j] * before;
      Kd[o] = k[j] * x;
      Qd[o] = q[j] * x;
      Kw[o] = k[j] * (suf[j] * behind);
    }
    if (sub == 0) E[(static_cast<size_t>(chunk) * a.H + head) * dk + ch] = pre[15] * behind;
  }
  __syncthreads();
  // the diagonal blocks' inverses: lane c column c (forward substitution)
  for (int b = wave; b < RT; b += WAVES) {
    const float* L = Ls + (16 * b) * TLD + 16 * b;
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == l16 ? 1.f : 0.f;
#pragma unroll
      for (int c = 0; c < r; ++c) v = fmaf(-L[r * TLD + c], x[c], v);
      x[r] = v;
    }
    if (lq == 0) {
#pragma unroll
      for (int r = 0; r < 16; ++r) Ts[(16 * b + r) * TLD + 16 * b + l16] = x[r];
    }
  }
  __syncthreads();
  // T_ij = -T_ii (sum over j <= m < i of L_im T_mj), one block diagonal after the other
  for (int d = 1; d < RT; ++d) {
    for (int j = wave; d + j < RT; j += WAVES) {
      const int i = d + j;
      f32x4 p = zero4();
      for (int m = j; m < i; ++m) {
        const f32x4 a4 = *reinterpret_cast<const f32x4*>(Ls + (16 * i + l16) * TLD + 16 * m + 4 * lq);
        const float* t4 = Ts + (16 * m + 4 * lq) * TLD + 16 * j + l16;
#pragma unroll
        for (int e = 0; e < 4; ++e) p = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[e], t4[e * TLD], p, 0, 0, 0);
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
  for (int i = tid; i < CL * CL; i += NT) {
    const int t = i / CL, c = i - t * CL;
    if (c / 16 <= t / 16) T[mat + i] = Ts[t * TLD + c] * sw[c];
  }
}

struct RowArgs {
  int ld, dk;
};

// runs: rows (sequence, first chunk, chunks).  Workgroup (head, 16 value columns, run): the heads are the grid's
// fastest index, so with eight heads or a multiple the slices of a head, which read the same Kd, Kw and T, lie on
// one XCD and find them in its L2.  A chunk's Kd, Kw, T, V
// and P(0, L) are asked for while the chunk before is worked on.  W [chunks, H, dk, dv] receives the state
// before every chunk, U [tokens, H, dv] the chunks' u.
constexpr int DCOLS = 16;
template <int DKP, int CL> constexpr size_t delta_lds() {
  return 4 * (DKP + 2 * CL * (DKP + 4) + CL * (CL + 4) + 3 * DCOLS * (CL + 4) + DCOLS * (DKP + 4));
}
template <int DKP, int CL, bool VEC>
__global__ __launch_bounds__(256) void chdelta_delta_kernel(
    const float* __restrict__ rows, const int* __restrict__ chunks, const int* __restrict__ runs,
    const int* __restrict__ positions, const int* __restrict__ slot_ids, float* __restrict__ state,
    const float* __restrict__ T, const float* __restrict__ E, const float* __restrict__ Kd, const float* __restrict__ Kw,
    float* __restrict__ W, float* __restrict__ U, ChArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4, RT = CL / 16;
  float* el = lds;                               // [DKP] P(0, L)
  float* Kds = el + DKP;                         // [CL][QLD]
  float* Kws = Kds + CL * QLD;                   // [CL][QLD]
  float* Tb = Kws + CL * QLD;                    // [CL][TLD]
  float* Vt = Tb + CL * TLD;                     // [DCOLS][TLD]
  float* Rt = Vt + DCOLS * TLD;                  // [DCOLS][TLD]
  float* Ut = Rt + DCOLS * TLD;                  // [DCOLS][TLD]
  float* St = Ut + DCOLS * TLD;                  // [DCOLS][QLD]
  const int head = blockIdx.x, col0 = blockIdx.y * DCOLS;
  const int seq = runs[3 * blockIdx.z], c0 = runs[3 * blockIdx.z + 1], nc = runs[3 * blockIdx.z + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int dk = a.dk, dv = a.dv;
  int slot = slot_ids[seq];
  if (slot < 0 || slot >= a.n_slots) slot = -1;
  float* S_slot = slot >= 0 ? state + static_cast<size_t>(slot) * a.slot_stride + static_cast<size_t>(head) * dk * dv
                            : nullptr;
  const bool resume = slot >= 0 && positions[chunks[4 * c0 + 1]] > 0;
  for (int i = tid; i < DKP * DCOLS; i += 256) {
    const int r = i / DCOLS, cl = i % DCOLS, c = col0 + cl;
    St[cl * QLD + r] = (resume && r < dk && c < dv) ? S_slot[static_cast<size_t>(r) * dv + c] : 0.f;
  }
  const RowArgs ka{a.H * dk, dk};
  const int k_off = head * dk, v_off = a.v_off + head * dv;
  constexpr int NT = CL * CL / 4 / 256;
  StagedRows<DKP, CL, 256, VEC> kd, kw;
  StagedTurned<CL, DCOLS, 256, TLD> vs;
  f32x4 treg[NT];
  float ereg = 0.f;
  auto ask = [&](int ch, int tb, int cnt) {
    kd.ask(Kd, ka, k_off, tb, cnt);
    kw.ask(Kw, ka, k_off, tb, cnt);
    const float* Tg = T + (static_cast<size_t>(ch) * a.H + head) * CL * CL;
#pragma unroll
    for (int x = 0; x < NT; ++x) treg[x] = *reinterpret_cast<const f32x4*>(Tg + 4 * (tid + 256 * x));
    vs.ask(rows + static_cast<size_t>(tb) * a.ld + v_off + col0, a.ld, cnt, dv - col0);
    ereg = E[(static_cast<size_t>(ch) * a.H + head) * dk + min(tid, dk - 1)];
  };
  int tb = chunks[4 * c0 + 1], cnt = chunks[4 * c0 + 2];
  ask(c0, tb, cnt);
  for (int j = 0; j < nc; ++j) {
    const int ch = c0 + j;
    // the next chunk's place, asked for early
    const int tb_next = j + 1 < nc ? chunks[4 * (ch + 1) + 1] : 0, cnt_next = j + 1 < nc ? chunks[4 * (ch + 1) + 2] : 0;
    __syncthreads();   // the chunk before is done with everything
    kd.put(Kds, cnt, dk);
    kw.put(Kws, cnt, dk);
#pragma unroll
    for (int x = 0; x < NT; ++x)
      *reinterpret_cast<f32x4*>(Tb + (4 * tid / CL + x * (1024 / CL)) * TLD + 4 * tid % CL) = treg[x];
    vs.put(Vt, cnt, dv - col0);
    if (tid < DKP) el[tid] = ereg;
    __syncthreads();
    if (j + 1 < nc) ask(ch + 1, tb_next, cnt_next);
    // R = V - Kd S
    if (wave < RT) {
      const f32x4 acc = mma_rows<DKP>(Kds + (16 * wave + l16) * QLD + 4 * lq, St + l16 * QLD + 4 * lq, zero4());
      const int t = 16 * wave + 4 * lq;
      *reinterpret_cast<f32x4*>(Rt + l16 * TLD + t) = *reinterpret_cast<const f32x4*>(Vt + l16 * TLD + t) - acc;
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
      *reinterpret_cast<f32x4*>(Ut + l16 * TLD + t) = u;
#pragma unroll
      for (int v = 0; v < 4; ++v)
        if (t + v < cnt && c < dv) U[(static_cast<size_t>(tb + t + v) * a.H + head) * dv + c] = u[v];
    }
    __syncthreads();
    // S <- P(0, L) S + Kw^T U; the state as it was goes to W
    float* Wg = W + (static_cast<size_t>(ch) * a.H + head) * dk * dv;
    f32x4 b4[RT];
#pragma unroll
    for (int k = 0; k < RT; ++k) b4[k] = *reinterpret_cast<const f32x4*>(Ut + l16 * TLD + 16 * k + 4 * lq);
    for (int kt = wave; kt < DKP / 16; kt += 4) {
      f32x4* mine = reinterpret_cast<f32x4*>(St + l16 * QLD + 16 * kt + 4 * lq);
      const float* kp = Kws + (4 * lq) * QLD + 16 * kt + l16;
      float kv[RT][4];
#pragma unroll
      for (int k = 0; k < RT; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) kv[k][e] = kp[(16 * k + e) * QLD];
      const f32x4 old = *mine;
      f32x4 acc = old * *reinterpret_cast<const f32x4*>(el + 16 * kt + 4 * lq);
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

// Workgroup of eight waves (head, 64 value columns, chunk): O = A U + Qd S0.  Wave w has the chunk's rows
// 16 (w % RT) .. + 15, whose Qd it keeps in registers.
constexpr int VCOLS = 64;
template <int DKP, int CL> constexpr size_t read_lds() {
  return 4 * (VCOLS * (DKP + 4) + CL * (CL + 4) + VCOLS * (CL + 4));
}
template <int DKP, int CL, bool VEC>
__global__ __launch_bounds__(512, DKP <= 128 ? 4 : 2) void chdelta_read_kernel(
    const int* __restrict__ chunks, const float* __restrict__ Qd, const float* __restrict__ A,
    const float* __restrict__ W, const float* __restrict__ U, float* __restrict__ out, ChArgs a) {
  extern __shared__ __align__(16) float lds[];
  constexpr int QLD = DKP + 4, TLD = CL + 4, RT = CL / 16, SHARES = 8 / RT, NA = (CL * CL / 4 + 511) / 512;
  float* Sc = lds;                               // [VCOLS][QLD] the state's columns
  float* As = Sc + VCOLS * QLD;                  // [CL][TLD]
  float* Ut = As + CL * TLD;                     // [VCOLS][TLD]
  const int chunk = blockIdx.z, head = blockIdx.x, col0 = blockIdx.y * VCOLS;
  const int tb = chunks[4 * chunk + 1], cnt = chunks[4 * chunk + 2];
  const int tid = threadIdx.x, lane = tid % KVF_WAVE, wave = tid / KVF_WAVE, l16 = lane % 16, lq = lane / 16;
  const int dk = a.dk, dv = a.dv, rt = wave % RT, share = wave / RT;
  StagedTurned<CL, VCOLS, 512, TLD> us;
  StagedTurned<DKP, VCOLS, 512, QLD> ws;
  us.ask(U + (static_cast<size_t>(tb) * a.H + head) * dv + col0, static_cast<size_t>(a.H) * dv, cnt, dv - col0);
  ws.ask(W + (static_cast<size_t>(chunk) * a.H + head) * dk * dv + col0, dv, dk, dv - col0);
  f32x4 areg[NA];
  const float* Ag = A + (static_cast<size_t>(chunk) * a.H + head) * CL * CL;
#pragma unroll
  for (int x = 0; x < NA; ++x) {
    const int i = 4 * (tid + 512 * x);
    areg[x] = *reinterpret_cast<const f32x4*>(Ag + (i < CL * CL ? i : 0));
  }
  f32x4 q4[DKP / 16];
  const bool q_ok = 16 * rt + l16 < cnt;
  {
    const float* p = Qd + (static_cast<size_t>(tb + 16 * rt + l16) * a.H + head) * dk;
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) q4[u] = load_four<VEC>(Qd, p, 16 * u + 4 * lq, dk, q_ok);
  }
  us.put(Ut, cnt, dv - col0);
  ws.put(Sc, dk, dv - col0);
#pragma unroll
  for (int x = 0; x < NA; ++x) {
    const int i = 4 * (tid + 512 * x);
    if (i < CL * CL) *reinterpret_cast<f32x4*>(As + (i / CL) * TLD + i % CL) = areg[x];
  }
#pragma unroll
  for (int u = 0; u < DKP / 16; ++u) q4[u] = clear_past(q4[u], 16 * u + 4 * lq, dk, q_ok);
  __syncthreads();
  const int col_tiles = min(VCOLS / 16, (dv - col0 + 15) / 16), t4 = 16 * rt + 4 * lq;
  for (int ct = share; ct < col_tiles; ct += SHARES) {
    f32x4 acc = zero4();
    const float* sb = Sc + (16 * ct + l16) * QLD + 4 * lq;
#pragma unroll
    for (int u = 0; u < DKP / 16; ++u) {
      const f32x4 b4 = *reinterpret_cast<const f32x4*>(sb + 16 * u);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[u][e], b4[e], acc, 0, 0, 0);
    }
    acc = mma_rows(As + (16 * rt + l16) * TLD + 4 * lq, Ut + (16 * ct + l16) * TLD + 4 * lq, 16 * (rt + 1), acc);
    const int c = col0 + 16 * ct + l16;
#pragma unroll
    for (int v = 0; v < 4; ++v)
      if (t4 + v < cnt && c < dv) out[(static_cast<size_t>(tb + t4 + v) * a.H + head) * dv + c] = acc[v];
  }
}

struct ChunkPtrs {
  const float *rows, *z, *zb, *neg_a, *dt_bias;
  const int *positions, *slot_ids, *chunks, *runs;
  float *state, *out, *T, *A, *E, *Kd, *Kw, *Qd, *W, *U;
  int n_chunks, n_runs;
};

template <int DKP, int CL, bool VEC> int chunks_go(const ChunkPtrs& p, ChArgs a, hipStream_t s) {
  static bool allowed = false;
  constexpr size_t lds_solve = solve_lds<DKP, CL>(), lds_delta = delta_lds<DKP, CL>(), lds_read = read_lds<DKP, CL>();
  if (!allowed) {
    hipError_t e = allow_lds(&chdelta_solve_kernel<DKP, CL>, lds_solve);
    if (e == hipSuccess) e = allow_lds(&chdelta_delta_kernel<DKP, CL, VEC>, lds_delta);
    if (e == hipSuccess) e = allow_lds(&chdelta_read_kernel<DKP, CL, VEC>, lds_read);
    if (e != hipSuccess) return static_cast<int>(e);
    allowed = true;
  }
  hipLaunchKernelGGL((chdelta_solve_kernel<DKP, CL>), dim3(a.H, p.n_chunks), dim3(solve_threads<DKP, CL>()), lds_solve, s,
                     p.rows, p.z, p.zb, p.neg_a, p.dt_bias, p.chunks, p.T, p.A, p.E, p.Kd, p.Kw, p.Qd, a);
  hipLaunchKernelGGL((chdelta_delta_kernel<DKP, CL, VEC>), dim3(a.H, (a.dv + DCOLS - 1) / DCOLS, p.n_runs), dim3(256),
                     lds_delta, s, p.rows, p.chunks, p.runs, p.positions, p.slot_ids, p.state, p.T, p.E, p.Kd, p.Kw, p.W,
                     p.U, a);
  hipLaunchKernelGGL((chdelta_read_kernel<DKP, CL, VEC>), dim3(a.H, (a.dv + VCOLS - 1) / VCOLS, p.n_chunks), dim3(512),
                     lds_read, s, p.chunks, p.Qd, p.A, p.W, p.U, p.out, a);
  return kvf_last_error();
}

bool args_ok(const ChArgs& a) {
  return a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.H <= 65535 && a.dk > 0 && a.dk <= 256 && a.dv > 0 &&
         a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.q_off + a.G * a.dk <= a.ld && a.k_off + a.G * a.dk <= a.ld &&
         a.v_off + a.H * a.dv <= a.ld && a.a_off >= 0 && a.a_off + a.H * a.dk <= a.z_ld && a.b_off >= 0 &&
         a.b_off + a.H <= a.b_ld && a.dv <= 65535 && static_cast<long>(a.slot_stride) >= static_cast<long>(a.H) * a.dk * a.dv;
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

KVF_EXPORT int kvf_chdelta_chunk_len(int dk) { return dk <= 128 ? 64 : 32; }

// The runs named in `runs` (sequence, first chunk, chunks), cut into `chunks` (sequence, first token, tokens, 0; at
// most kvf_chdelta_chunk_len(dk) tokens each, a run's chunks in order and one after another).  Scratch: T, A
// [n_chunks, H, CL, CL], E [n_chunks, H, dk], Kd, Kw, Qd [tokens, H, dk], W [n_chunks, H, dk, dv], U [tokens, H, dv],
// all on 16 bytes.
KVF_EXPORT int kvf_chdelta_chunks(CHDELTA_ARGS_DECL, const int* chunks, int n_chunks, const int* runs, int n_runs,
                                  float* T, float* A, float* E, float* Kd, float* Kw, float* Qd, float* W, float* U,
                                  hipStream_t s) {
  if (n_chunks <= 0 || n_runs <= 0) return 0;
  const ChArgs a{H, G, dk, dv, ld, q_off, k_off, v_off, z_ld, a_off, b_ld, b_off, n_slots, slot_stride, 0};
  if (!args_ok(a) || n_chunks > 65535 || n_runs > 65535 || !chunks || !runs || !T || !A || !E || !Kd || !Kw || !Qd || !W || !U)
    return static_cast<int>(hipErrorInvalidValue);
  const ChunkPtrs p{rows, z, zb, neg_a, dt_bias, positions, slot_ids, chunks, runs, state, out, T, A, E, Kd, Kw, Qd, W, U,
                    n_chunks, n_runs};
  const bool vec = dk % 4 == 0;
#define GO(DKP, CL) return vec ? chunks_go<DKP, CL, true>(p, a, s) : chunks_go<DKP, CL, false>(p, a, s)
  if (dk <= 32) GO(32, 64);
  if (dk <= 64) GO(64, 64);
  if (dk <= 128) GO(128, 64);
  GO(256, 32);
#undef GO
}
