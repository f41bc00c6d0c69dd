// What lies between the q/k/v projection and the paged attention kernels where the projected rows
// pass a short causal convolution over time first:
//     y_t[c] = sum_j w[c, j] x_(t - (taps-1) + j)[c]          (zeros before a sequence's first token)
// per channel c of q, k and v; then q and k heads may be divided by their root mean square over dk
// elements (and multiplied by weights that the heads share); q goes to rows of its own, k and v to
// the pages.  One kernel, fp32 from the projected row on, one rounding.  What lies before a run is
// taken from the sequence's state slot, [taps - 1][C] floats (the oldest first), where the run leaves
// its own last inputs.
//
// Channels come in heads of d (padded: elements dk .. d - 1 of a head have zero rows and weights and stay
// zero): H q heads, KV k heads, KV v heads.  P = 4 .. 64 lanes share a head, four neighbouring
// elements each.  A run is cut into tiles of TT tokens at multiples of TT *positions*, so that a
// tile's values lie side by side in one (transposed) V page where a page's size is a multiple of
// TT; a workgroup takes two tiles.  Only the first two tiles of a run can reach back into the slot
// (taps - 1 < TT), so they are one workgroup's, and each of its threads alone reads and rewrites the
// slot's numbers of its channels.  The weights lie [taps][C].
#include "common.h"

namespace {
struct CkArgs {
  int H, KV, d, dk, ld, ldq;             // rows [tokens, ld], q_out [tokens, ldq]
  int norm;                              // q and k heads are divided by their root mean square
  float eps;
  int bs, nb, table_stride, n_seqs;      // pages of bs tokens
  int n_slots, slot_stride;              // state [n_slots, slot_stride]
};

__device__ __forceinline__ void load4(const float* p, float (&v)[4]) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
__device__ __forceinline__ void load4(const bf16_t* p, float (&v)[4]) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(r.x << 16); v[1] = __uint_as_float(r.x & 0xffff0000u);
  v[2] = __uint_as_float(r.y << 16); v[3] = __uint_as_float(r.y & 0xffff0000u);
}
__device__ __forceinline__ void store4(float* p, const float (&v)[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ uint32_t two(float a, float b) {
  return static_cast<uint32_t>(f32_to_bf16(a)) | (static_cast<uint32_t>(f32_to_bf16(b)) << 16);
}
__device__ __forceinline__ void store4(bf16_t* p, const float (&v)[4]) {
  *reinterpret_cast<uint2*>(p) = make_uint2(two(v[0], v[1]), two(v[2], v[3]));
}
// TT neighbouring numbers of a column, y[0 .. TT-1][e]
template <int TT> __device__ __forceinline__ void store_run(float* p, const float (&y)[TT][4], int e) {
#pragma unroll
  for (int i = 0; i < TT; i += 4)
    *reinterpret_cast<float4*>(p + i) = make_float4(y[i][e], y[i + 1][e], y[i + 2][e], y[i + 3][e]);
}
template <int TT> __device__ __forceinline__ void store_run(bf16_t* p, const float (&y)[TT][4], int e) {
#pragma unroll
  for (int i = 0; i < TT; i += 8)
    *reinterpret_cast<uint4*>(p + i) = make_uint4(two(y[i][e], y[i + 1][e]), two(y[i + 2][e], y[i + 3][e]),
                                                  two(y[i + 4][e], y[i + 5][e]), two(y[i + 6][e], y[i + 7][e]));
}

// Grid (shares of the heads, pairs of tiles, sequences).  TT = 1: every run of the launch is one token.
template <typename T, int TAPS, int TT>
__global__ __launch_bounds__(256) void conv_norm_kvwrite_kernel(
    const T* __restrict__ rows, const float* __restrict__ w, const float* __restrict__ qw, const float* __restrict__ kw,
    const int* __restrict__ cu_q, const int* __restrict__ positions, const int* __restrict__ slot_ids,
    const int* __restrict__ block_table, float* __restrict__ state, T* __restrict__ q_out, T* __restrict__ k_pages,
    T* __restrict__ v_pages, int P, CkArgs a) {
  constexpr int K = TAPS - 1;
  const int seq = blockIdx.z;
  const int run0 = cu_q[seq], run1 = cu_q[seq + 1], len = run1 - run0;
  if (len <= 0) return;
  const int p0 = positions[run0];
  const int lead = TT > 1 && p0 > 0 ? p0 % TT : 0;          // positions of the first tile that lie before the run
  const int first_tile = 2 * blockIdx.y, last_tile = first_tile + 1;
  if (first_tile * TT - lead >= len) return;
  const int group = threadIdx.x / P, lane = threadIdx.x % P;
  const int head = blockIdx.x * (256 / P) + group;          // of H + 2 KV
  const bool ok = head < a.H + 2 * a.KV && 4 * lane < a.d;  // (idle lanes read what the first head's lanes read)
  const int C = (a.H + 2 * a.KV) * a.d;
  const int c = ok ? head * a.d + 4 * lane : 0;
  const T* src = rows + c;
  float wt[TAPS][4];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) load4(w + static_cast<size_t>(j) * C + c, wt[j]);
  float old[K > 0 ? K : 1][4] = {};
  float* st = nullptr;
  if (K > 0 && blockIdx.y == 0) {
    const int slot = slot_ids[seq];
    if (slot >= 0 && slot < a.n_slots) {
      st = state + static_cast<size_t>(slot) * a.slot_stride + c;
      if (p0 > 0) {
#pragma unroll
        for (int j = 0; j < K; ++j) load4(st + static_cast<size_t>(j) * C, old[j]);
      }
    }
  }
  const bool is_q = head < a.H, is_v = head >= a.H + a.KV;
  const int kvh = is_q ? 0 : (head - a.H) % (a.KV > 0 ? a.KV : 1);
  const float* nw = is_q ? qw : kw;
  const int* table = block_table + static_cast<size_t>(seq) * a.table_stride;
  for (int tile = first_tile; tile <= last_tile; ++tile) {
    const int i0 = max(0, tile * TT - lead), i1 = min(len, (tile + 1) * TT - lead);   // tokens of the run
    if (i0 >= i1) break;
    const int cnt = i1 - i0;
    float x[TT + K][4];                                     // x[K + i] is the run's token i0 + i
#pragma unroll
    for (int j = 0; j < K; ++j) {
      const int i = i0 - K + j;
      if (i >= 0) {
        load4(src + static_cast<size_t>(run0 + i) * a.ld, x[j]);
      } else {
        // input number K + i of the slot's (a tile that starts behind the run's first K tokens has none)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float v = 0.f;
#pragma unroll
          for (int o = 0; o < K; ++o) v = K + i == o ? old[o][e] : v;
          x[j][e] = v;
        }
      }
    }
    // (past the tile's end its last row is read again and not used, so that no load is predicated)
#pragma unroll
    for (int i = 0; i < TT; ++i) load4(src + static_cast<size_t>(run0 + i0 + min(i, cnt - 1)) * a.ld, x[K + i]);
    float y[TT][4];
#pragma unroll
    for (int i = 0; i < TT; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float acc = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) acc = fmaf(wt[j][e], x[i + j][e], acc);
        y[i][e] = acc;
      }
    }
    if (a.norm) {   // the same for all lanes: the lanes of a head add up their squares
#pragma unroll
      for (int i = 0; i < TT; ++i) {
        float ss = 0.f;
        if (ok)
          ss = fmaf(y[i][0], y[i][0], fmaf(y[i][1], y[i][1], fmaf(y[i][2], y[i][2], y[i][3] * y[i][3])));
        for (int o = P / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, KVF_WAVE);
        const float r = is_v ? 1.f : 1.f / sqrtf(ss / static_cast<float>(a.dk) + a.eps);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          y[i][e] *= r;
          if (nw && !is_v && ok) y[i][e] *= 4 * lane + e < a.dk ? nw[4 * lane + e] : 0.f;
        }
      }
    }
    if (ok && is_q) {
#pragma unroll
      for (int i = 0; i < TT; ++i)
        if (i < cnt) store4(q_out + static_cast<size_t>(run0 + i0 + i) * a.ldq + c, y[i]);
    } else if (ok) {
      const int p = p0 + i0;
      bool whole = false;
      if (TT > 1 && is_v && cnt == TT && a.bs % TT == 0 && p >= 0) {   // p is a multiple of TT here
        const int blk = p / a.bs;
        const int page = blk < a.table_stride ? table[blk] : -1;
        whole = true;
        if (page >= 0 && page < a.nb) {
          T* dst = v_pages + ((static_cast<size_t>(page) * a.KV + kvh) * a.d + 4 * lane) * a.bs + (p - blk * a.bs);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if constexpr (TT > 1) store_run<TT>(dst + static_cast<size_t>(e) * a.bs, y, e);
        }
      }
      if (!whole) {
#pragma unroll
        for (int i = 0; i < TT; ++i) {
          if (i >= cnt || p + i < 0) continue;
          const int blk = (p + i) / a.bs, off = (p + i) - blk * a.bs;
          const int page = blk < a.table_stride ? table[blk] : -1;
          if (page < 0 || page >= a.nb) continue;
          if (is_v) {
            T* dst = v_pages + ((static_cast<size_t>(page) * a.KV + kvh) * a.d + 4 * lane) * a.bs + off;
#pragma unroll
            for (int e = 0; e < 4; ++e) Elem<T>::store(dst + static_cast<size_t>(e) * a.bs, y[i][e]);
          } else {
            store4(k_pages + ((static_cast<size_t>(page) * a.KV + kvh) * a.bs + off) * a.d + 4 * lane, y[i]);
          }
        }
      }
    }
  }
  if (st != nullptr && ok) {
    // the last K inputs of (old ones, this run): entry j is input number len + j
    float keep[K > 0 ? K : 1][4];
#pragma unroll
    for (int j = 0; j < K; ++j) {
      const int i = len + j;                                // < K: an old input
      if (i >= K) {
        load4(src + static_cast<size_t>(run0 + i - K) * a.ld, keep[j]);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float v = 0.f;
#pragma unroll
          for (int o = 0; o < K; ++o) v = i == o ? old[o][e] : v;
          keep[j][e] = v;
        }
      }
    }
#pragma unroll
    for (int j = 0; j < K; ++j) store4(st + static_cast<size_t>(j) * C, keep[j]);
  }
}

constexpr int TILE = 8;

template <typename T, int TAPS>
int go(const void* rows, const float* w, const float* qw, const float* kw, const int* cu_q, const int* positions,
       const int* slot_ids, const int* block_table, float* state, void* q_out, void* k_pages, void* v_pages, int longest,
       CkArgs a, hipStream_t s) {
  int P = 4;
  while (4 * P < a.d) P *= 2;
  const int shares = (a.H + 2 * a.KV + 256 / P - 1) / (256 / P);
  const int tiles = longest == 1 ? 1 : (longest + TILE - 1 + TILE - 1) / TILE;
#define GO(TT)                                                                                                        \
  hipLaunchKernelGGL((conv_norm_kvwrite_kernel<T, TAPS, TT>), dim3(shares, (tiles + 1) / 2, a.n_seqs),               \
                     dim3(256), 0, s, static_cast<const T*>(rows), w, qw, kw, cu_q, positions, slot_ids, block_table, \
                     state, static_cast<T*>(q_out), static_cast<T*>(k_pages), static_cast<T*>(v_pages), P, a)
  if (longest == 1) GO(1);
  else GO(TILE);
#undef GO
  return kvf_last_error();
}
}  // namespace

// dtype: 0 = fp32, 1 = bf16 (rows, q_out and pages).  rows [n, ld]: (H + 2 KV) heads of d; w [taps, (H + 2 KV) d]
// fp32; qw, kw: null, or [dk] fp32 (with norm).  longest: tokens of the longest run.  ld, ldq, slot_stride and d are
// multiples of 4, and rows, q_out, pages and state start on 16 bytes (what the host checks).
KVF_EXPORT int kvf_conv_norm_kvwrite(int dtype, const void* rows, int ld, int taps, const float* w, int norm, int dk,
                                     float eps, const float* qw, const float* kw, const int* cu_q, const int* positions,
                                     const int* slot_ids, const int* block_table, int table_stride, float* state,
                                     int n_slots, int slot_stride, void* q_out, int ldq, void* k_pages, void* v_pages,
                                     int H, int KV, int d, int bs, int nb, int n_seqs, int longest, hipStream_t s) {
  if (n_seqs <= 0 || longest <= 0) return 0;
  if (H <= 0 || KV <= 0 || d <= 0 || d % 16 || d > 256 || dk <= 0 || dk > d || ld % 4 || ldq % 4 || ldq < H * d ||
      ld < (H + 2 * KV) * d || bs <= 0 || nb <= 0 || n_seqs > 65535 || taps < 1 || taps > TILE ||
      (taps > 1 && (!state || slot_stride % 4 || static_cast<long>(taps - 1) * (H + 2 * KV) * d > slot_stride)) ||
      (longest + 2 * TILE) / TILE > 65535)
    return static_cast<int>(hipErrorInvalidValue);
  const CkArgs a{H, KV, d, dk, ld, ldq, norm, eps, bs, nb, table_stride, n_seqs, n_slots, slot_stride};
#define CASE(N)                                                                                                      \
  case N:                                                                                                            \
    return dtype == 0 ? go<float, N>(rows, w, qw, kw, cu_q, positions, slot_ids, block_table, state, q_out, k_pages, \
                                     v_pages, longest, a, s)                                                         \
                      : go<bf16_t, N>(rows, w, qw, kw, cu_q, positions, slot_ids, block_table, state, q_out, k_pages, \
                                      v_pages, longest, a, s)
  if (dtype != 0 && dtype != 1) return static_cast<int>(hipErrorInvalidValue);
  switch (taps) {
    CASE(1); CASE(2); CASE(3); CASE(4); CASE(5); CASE(6); CASE(7); CASE(8);
  }
#undef CASE
  return static_cast<int>(hipErrorInvalidValue);
}
