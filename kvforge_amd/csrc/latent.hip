// Latent attention: what lies between the projections and the paged attention kernels.
//
// A token's keys and values of all heads are read out of one latent vector c [rank] (RMS-normed)
// and one rotated key part k_r [rot] that the heads share.  With W_uk the read-out of the
// unrotated keys, q_h . (W_uk_h c) = (W_uk_h^T q_h) . c, so attention runs over ONE key per
// token, [k_r | c], with per-head queries [q_r_h | W_uk_h^T q_h]; the weighted sum of the c is
// taken by the same kernels (the value is the key's c part) and read out per head by W_uv_h
// afterwards.  The cache holds k_r and c and nothing per head.
//
//   latent_split : a token's projected rows [q heads (dim | rot) ...] and [c_raw (rank) | k_r (rot)] become
//                  the attention kernels' row [H q heads | k | v] of heads of d elements:
//                  q head h = [q_r_h | (left for head_product) | 0], k = [k_r | norm(c) | 0],
//                  v = [0 | norm(c) | 0]; the norm in fp32 with one rounding.  Without a norm
//                  weight the row holds the q heads alone (attention over another layer's keys).
//   head_product : out[n, h, :] = W[h] in[n, h, :] for per-head matrices W [H, O, I].  bf16 rows and
//                  weights whose heads start on 16 bytes go to the matrix cores (a workgroup
//                  per 64 rows x 64 outputs of a head, a wave per 16 outputs, operands straight
//                  from memory, fp32 sums); everything else is fp32 multiply and add on the
//                  vector ALUs, tiles of 32 rows x 64 outputs through LDS.  With `gate` (rows of
//                  one number per head) what is stored is the product times sigmoid(gate[n, h]), or
//                  with a number per output (ELEM) times sigmoid(gate[n, h * O + o]); and times `scale`.
//   latent_norm  : an RMS norm of a block of a row's columns (the queries' latent), out in rows of its own.
#include "common.h"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void latent_split_kernel(const T* __restrict__ q, int ld_q,
                                                           const T* __restrict__ downs, int ld_down,
                                                           T* __restrict__ qkv, int ld_out,
                                                           const float* __restrict__ w, float eps, int H,
                                                           int dim, int rot, int rank, int d) {
  __shared__ float scratch[16];
  const int n = blockIdx.x, tid = threadIdx.x;
  const T* in = q + static_cast<size_t>(n) * ld_q;
  T* out = qkv + static_cast<size_t>(n) * ld_out;
  const T* down = downs + static_cast<size_t>(n) * ld_down;
  // few tokens: a token's heads are shared among workgroups, of which the first has the key and value
  const int h0 = static_cast<int>(static_cast<long>(H) * blockIdx.y / gridDim.y);
  const int h1 = static_cast<int>(static_cast<long>(H) * (blockIdx.y + 1) / gridDim.y);
  const bool own = w != nullptr && blockIdx.y == 0;
  float r = 0.f;
  if (own) {   // the same for the whole workgroup
    float ss = 0.f;
    for (int i = tid; i < rank; i += blockDim.x) {
      const float v = Elem<T>::load(down + i);
      ss = fmaf(v, v, ss);
    }
    r = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(rank) + eps);
  }
  // q heads: the rotated part to the front, zeros behind what head_product fills
  for (int i = h0 * d + tid; i < h1 * d; i += blockDim.x) {
    const int h = i / d, e = i - h * d;
    if (e < rot)
      out[i] = in[h * (dim + rot) + dim + e];
    else if (e >= rot + rank || dim == 0)   // (heads without a plain part: nothing fills the middle)
      Elem<T>::store(out + i, 0.f);
  }
  if (!own) return;
  T* k = out + H * d;
  T* v = k + d;
  for (int e = tid; e < d; e += blockDim.x) {
    if (e < rot) {
      k[e] = down[rank + e];
      Elem<T>::store(v + e, 0.f);
    } else if (e < rot + rank) {
      const float c = Elem<T>::load(down + e - rot) * r * w[e - rot];
      Elem<T>::store(k + e, c);
      Elem<T>::store(v + e, c);
    } else {
      Elem<T>::store(k + e, 0.f);
      Elem<T>::store(v + e, 0.f);
    }
  }
}

// out[n, :] = in[n, :rank] / sqrt(mean(in^2) + eps) * w in fp32, one rounding; a workgroup per row.  VEC: rows start
// on 16 / 32 bytes and rank is a multiple of eight, eight neighbours a load.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void latent_norm_kernel(const T* __restrict__ in, int ld_in, const float* __restrict__ w,
                                                          float eps, T* __restrict__ out, int rank) {
  __shared__ float scratch[16];
  constexpr int V = VEC ? 8 : 1;
  const T* x = in + static_cast<size_t>(blockIdx.x) * ld_in;
  T* o = out + static_cast<size_t>(blockIdx.x) * rank;
  auto take = [&](int i, float (&v)[V]) {
    if constexpr (VEC) load8(x + i, v);
    else v[0] = Elem<T>::load(x + i);
  };
  float first[V];            // what a thread keeps (the rest of a long row is read again)
  float ss = 0.f;
  const int i0 = V * threadIdx.x, step = V * blockDim.x;
  if (i0 < rank) take(i0, first);
  for (int i = i0; i < rank; i += step) {
    float v[V];
    if (i != i0) take(i, v);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float u = i == i0 ? first[e] : v[e];
      ss = fmaf(u, u, ss);
    }
  }
  const float r = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(rank) + eps);
  for (int i = i0; i < rank; i += step) {
    float v[V];
    if (i != i0) take(i, v);
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = (i == i0 ? first[e] : v[e]) * r * w[i + e];
    if constexpr (VEC) {
      if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<float4*>(o + i) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(o + i + 4) = make_float4(v[4], v[5], v[6], v[7]);
      } else {
        uint32_t p[4];
#pragma unroll
        for (int e = 0; e < 4; ++e)
          p[e] = static_cast<uint32_t>(f32_to_bf16(v[2 * e])) | (static_cast<uint32_t>(f32_to_bf16(v[2 * e + 1])) << 16);
        *reinterpret_cast<uint4*>(o + i) = make_uint4(p[0], p[1], p[2], p[3]);
      }
    } else {
      Elem<T>::store(o + i, v[0]);
    }
  }
}

// the outputs' gate: rows of `ld` numbers (null: none), one per head or (ELEM kernels) one per output
template <typename T> struct HeadGate {
  const T* p;
  int ld;
  float scale;
};
template <typename T> __device__ __forceinline__ float gate_of(const HeadGate<T>& g, int n, int i) {
  return g.p ? g.scale / (1.f + expf(-Elem<T>::load(g.p + static_cast<size_t>(n) * g.ld + i))) : g.scale;
}

constexpr int HP_M = 32, HP_N = 64, HP_K = 32;

// grid (row tiles, output tiles, heads); 256 threads, thread (ty, tx) owns rows ty, ty + 16 and
// outputs tx + 16 j (j = 0..3) of the tile.
template <typename T, typename TW>
__global__ __launch_bounds__(256) void head_product_kernel(const T* __restrict__ in, int ld_in, int in_head,
                                                           const TW* __restrict__ W, T* __restrict__ out,
                                                           int ld_out, int out_head, int N, int O, int I,
                                                           HeadGate<T> gate, bool elem) {
  __shared__ float As[HP_M][HP_K + 1];
  __shared__ float Bs[HP_N][HP_K + 1];
  const int n0 = blockIdx.x * HP_M, o0 = blockIdx.y * HP_N, h = blockIdx.z;
  const int tid = threadIdx.x, ty = tid / 16, tx = tid % 16;
  const T* a = in + static_cast<size_t>(h) * in_head;
  const TW* w = W + static_cast<size_t>(h) * O * I;
  float acc[2][4] = {};
  for (int k0 = 0; k0 < I; k0 += HP_K) {
    for (int i = tid; i < HP_M * HP_K; i += 256) {
      const int r = i / HP_K, c = i % HP_K;
      As[r][c] = (n0 + r < N && k0 + c < I) ? Elem<T>::load(a + static_cast<size_t>(n0 + r) * ld_in + k0 + c) : 0.f;
    }
    for (int i = tid; i < HP_N * HP_K; i += 256) {
      const int r = i / HP_K, c = i % HP_K;
      Bs[r][c] = (o0 + r < O && k0 + c < I) ? Elem<TW>::load(w + static_cast<size_t>(o0 + r) * I + k0 + c) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < HP_K; ++c) {
      const float a0 = As[ty][c], a1 = As[ty + 16][c];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float b = Bs[tx + 16 * j][c];
        acc[0][j] = fmaf(a0, b, acc[0][j]);
        acc[1][j] = fmaf(a1, b, acc[1][j]);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int n = n0 + ty + 16 * i;
    if (n >= N) continue;
    T* o = out + static_cast<size_t>(n) * ld_out + static_cast<size_t>(h) * out_head;
    const float g = elem ? 1.f : gate_of(gate, n, h);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int e = o0 + tx + 16 * j;
      if (e < O) Elem<T>::store(o + e, acc[i][j] * (elem ? gate_of(gate, n, h * O + e) : g));
    }
  }
}

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

// a lane's four neighbouring outputs: one 8-byte store where the output rows allow it (`wide`:
// every head's outputs start on 8 bytes) and all four lie inside the head, else one by one
__device__ __forceinline__ void store4(bf16_t* o, const f32x4& a, int left, bool wide) {
  if (wide && left >= 4) {
    uint2 p;
    p.x = static_cast<unsigned>(f32_to_bf16(a[0])) | (static_cast<unsigned>(f32_to_bf16(a[1])) << 16);
    p.y = static_cast<unsigned>(f32_to_bf16(a[2])) | (static_cast<unsigned>(f32_to_bf16(a[3])) << 16);
    *reinterpret_cast<uint2*>(o) = p;
    return;
  }
#pragma unroll
  for (int v = 0; v < 4; ++v)
    if (v < left) Elem<bf16_t>::store(o + v, a[v]);
}

// a lane's four neighbouring outputs o .. o + 3 of head h times their gates (a row's gates that start on
// eight bytes are one load)
template <bool ELEM>
__device__ __forceinline__ f32x4 gated4(f32x4 a, const HeadGate<bf16_t>& g, float head_gate, int n, int h, int O, int o) {
  if constexpr (!ELEM) {
    return a * head_gate;
  } else {
    const bf16_t* p = g.p + static_cast<size_t>(n) * g.ld + static_cast<size_t>(h) * O + o;
    float z[4];
    if (o + 4 <= O && reinterpret_cast<uintptr_t>(p) % 8 == 0) {
      const uint2 r = *reinterpret_cast<const uint2*>(p);
      z[0] = __uint_as_float(r.x << 16); z[1] = __uint_as_float(r.x & 0xffff0000u);
      z[2] = __uint_as_float(r.y << 16); z[3] = __uint_as_float(r.y & 0xffff0000u);
    } else {
#pragma unroll
      for (int v = 0; v < 4; ++v) z[v] = o + v < O ? bf16_to_f32(p[v].bits) : 0.f;
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) a[v] *= g.scale / (1.f + __expf(-z[v]));
    return a;
  }
}

// v_mfma_f32_16x16x32_bf16 computes D[i][j] += sum_k A[i][k] B[j][k]; lane 16 c + r gives row r,
// elements 8c..8c+7 of the step's 32 of either operand, and holds D[4 (l / 16) + v][l % 16].
// A: 16 rows of the head's matrix (outputs), B: 16 rows of the input.  Grid (tiles of 64 rows,
// tiles of 64 outputs, heads); wave w takes outputs 16w..16w+15 of the tile for all its rows, so a
// weight fragment is loaded once for up to four row fragments.  I, in_head and ld_in are
// multiples of 8 and both bases lie on 16 bytes (the host checks), so a fragment is one 16-byte
// load that lies inside its row or is left zero.
template <bool ELEM>
__global__ __launch_bounds__(256) void head_product_mfma_kernel(const bf16_t* __restrict__ in, int ld_in,
                                                                int in_head, const bf16_t* __restrict__ W,
                                                                bf16_t* __restrict__ out, int ld_out, int out_head,
                                                                int N, int O, int I, bool wide,
                                                                HeadGate<bf16_t> gate) {
  const int n0 = blockIdx.x * 64, h = blockIdx.z;
  const int lane = threadIdx.x % KVF_WAVE, wave = threadIdx.x / KVF_WAVE;
  const int j = lane % 16, c = lane / 16;
  const int o0 = blockIdx.y * 64 + wave * 16;
  if (o0 >= O) return;
  const int subs = min(4, (N - n0 + 15) / 16);
  const bf16_t* wrow = o0 + j < O ? W + (static_cast<size_t>(h) * O + o0 + j) * I + 8 * c : nullptr;
  const bf16_t* xr[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int n = n0 + 16 * r + j;
    xr[r] = (r < subs && n < N) ? in + static_cast<size_t>(n) * ld_in + static_cast<size_t>(h) * in_head + 8 * c
                                : nullptr;
  }
  f32x4 acc[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < I; k0 += 32) {
    const bool inside = k0 + 8 * c + 8 <= I;
    uint4 wf = make_uint4(0u, 0u, 0u, 0u);
    if (wrow && inside) wf = *reinterpret_cast<const uint4*>(wrow + k0);
    uint4 xf[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      xf[r] = make_uint4(0u, 0u, 0u, 0u);
      if (xr[r] && inside) xf[r] = *reinterpret_cast<const uint4*>(xr[r] + k0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (r < subs)
        acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf),
                                                         __builtin_bit_cast(bf16x8, xf[r]), acc[r], 0, 0, 0);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int n = n0 + 16 * r + j;
    if (r >= subs || n >= N) continue;
    bf16_t* o = out + static_cast<size_t>(n) * ld_out + static_cast<size_t>(h) * out_head + o0 + 4 * c;
    store4(o, gated4<ELEM>(acc[r], gate, ELEM ? 1.f : gate_of(gate, n, h), n, h, O, o0 + 4 * c), O - (o0 + 4 * c), wide);
  }
}

// The same for many rows: a workgroup takes 64 rows of a head and ALL its outputs.  The rows'
// fragments (KS steps of 32 elements cover I) are loaded once and stay in registers while the
// wave goes through its groups of 16 outputs (w, w + 4, ...), so a row is read once per wave
// and not once per wave and output tile.  Sums run over the steps in the same order as above.
template <int KS, bool ELEM>
__global__ __launch_bounds__(256) void head_product_mfma_rows_kernel(const bf16_t* __restrict__ in, int ld_in,
                                                                     int in_head, const bf16_t* __restrict__ W,
                                                                     bf16_t* __restrict__ out, int ld_out,
                                                                     int out_head, int N, int O, int I, bool wide,
                                                                     HeadGate<bf16_t> gate) {
  const int n0 = blockIdx.x * 64, h = blockIdx.y;
  const int lane = threadIdx.x % KVF_WAVE, wave = threadIdx.x / KVF_WAVE;
  const int j = lane % 16, c = lane / 16;
  const int subs = min(4, (N - n0 + 15) / 16);
  uint4 xf[KS][4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int n = n0 + 16 * r + j;
    const bf16_t* x = (r < subs && n < N)
                          ? in + static_cast<size_t>(n) * ld_in + static_cast<size_t>(h) * in_head + 8 * c
                          : nullptr;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      xf[s][r] = make_uint4(0u, 0u, 0u, 0u);
      if (x && 32 * s + 8 * c + 8 <= I) xf[s][r] = *reinterpret_cast<const uint4*>(x + 32 * s);
    }
  }
  float gv[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) gv[r] = !ELEM && r < subs && n0 + 16 * r + j < N ? gate_of(gate, n0 + 16 * r + j, h) : 1.f;
  const int groups = (O + 15) / 16;
  for (int g = wave; g < groups; g += 4) {
    const int o0 = 16 * g;
    const bf16_t* wrow = o0 + j < O ? W + (static_cast<size_t>(h) * O + o0 + j) * I + 8 * c : nullptr;
    uint4 wf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      wf[s] = make_uint4(0u, 0u, 0u, 0u);
      if (wrow && 32 * s + 8 * c + 8 <= I) wf[s] = *reinterpret_cast<const uint4*>(wrow + 32 * s);
    }
    f32x4 acc[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KS; ++s)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (r < subs)
          acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf[s]),
                                                           __builtin_bit_cast(bf16x8, xf[s][r]), acc[r], 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = n0 + 16 * r + j;
      if (r >= subs || n >= N) continue;
      bf16_t* o = out + static_cast<size_t>(n) * ld_out + static_cast<size_t>(h) * out_head + o0 + 4 * c;
      store4(o, gated4<ELEM>(acc[r], gate, gv[r], n, h, O, o0 + 4 * c), O - (o0 + 4 * c), wide);
    }
  }
}

template <typename T, typename TW>
int head_product_launch(const void* in, int ld_in, int in_head, const void* W, void* out, int ld_out,
                        int out_head, int N, int H, int O, int I, const void* gate, int ld_gate, bool elem,
                        float scale, hipStream_t s) {
  const HeadGate<T> g{static_cast<const T*>(gate), ld_gate, scale};
  const dim3 grid((N + HP_M - 1) / HP_M, (O + HP_N - 1) / HP_N, H);
  hipLaunchKernelGGL((head_product_kernel<T, TW>), grid, dim3(256), 0, s, static_cast<const T*>(in), ld_in, in_head,
                     static_cast<const TW*>(W), static_cast<T*>(out), ld_out, out_head, N, O, I, g, elem);
  return kvf_last_error();
}

template <bool ELEM>
int head_product_mfma_launch(const bf16_t* x, int ld_in, int in_head, const bf16_t* w, bf16_t* y, int ld_out,
                             int out_head, int N, int H, int O, int I, bool wide, HeadGate<bf16_t> g, hipStream_t s) {
  const dim3 rows((N + 63) / 64, H);
#define ROWS(KS)                                                                                                     \
  hipLaunchKernelGGL((head_product_mfma_rows_kernel<KS, ELEM>), rows, dim3(256), 0, s, x, ld_in, in_head, w, y, ld_out, \
                     out_head, N, O, I, wide, g)
  if (N < 256 || I > 256) {   // few rows: more workgroups, each with one tile of outputs
    const dim3 grid((N + 63) / 64, (O + 63) / 64, H);
    hipLaunchKernelGGL((head_product_mfma_kernel<ELEM>), grid, dim3(256), 0, s, x, ld_in, in_head, w, y, ld_out, out_head,
                       N, O, I, wide, g);
  } else if (I <= 64) {
    ROWS(2);
  } else if (I <= 128) {
    ROWS(4);
  } else if (I <= 192) {
    ROWS(6);
  } else {
    ROWS(8);
  }
#undef ROWS
  return kvf_last_error();
}
}  // namespace

// out [n, rank] = RMS norm of in[:, :rank] (rows ld_in apart) times w; dtype of both: 0 = fp32, 1 = bf16.
KVF_EXPORT int kvf_latent_norm(int dtype, const void* in, int ld_in, const float* w, float eps, void* out, int n,
                               int rank, hipStream_t s) {
  if (n <= 0) return 0;
  if (rank <= 0 || ld_in < rank) return static_cast<int>(hipErrorInvalidValue);
  const size_t bytes = dtype == 0 ? 32 : 16;
  const bool vec = rank % 8 == 0 && ld_in % 8 == 0 && reinterpret_cast<uintptr_t>(in) % bytes == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  int threads = ((vec ? rank / 8 : rank) + KVF_WAVE - 1) / KVF_WAVE * KVF_WAVE;
  if (threads > 256) threads = 256;
#define GO(T, VEC)                                                                                                \
  hipLaunchKernelGGL((latent_norm_kernel<T, VEC>), dim3(n), dim3(threads), 0, s, static_cast<const T*>(in), ld_in, w, \
                     eps, static_cast<T*>(out), rank)
  if (dtype == 0) {
    if (vec) GO(float, true);
    else GO(float, false);
  } else if (dtype == 1) {
    if (vec) GO(bf16_t, true);
    else GO(bf16_t, false);
  } else {
    return static_cast<int>(hipErrorInvalidValue);
  }
#undef GO
  return kvf_last_error();
}

// dtype: 0 = fp32, 1 = bf16 (rows in and out).  d >= rot + rank.  w null: q heads alone.
KVF_EXPORT int kvf_latent_split(int dtype, const void* q, int ld_q, const void* down, int ld_down, void* qkv, int ld_out,
                                const float* w, float eps, int n, int H, int dim, int rot, int rank, int d, hipStream_t s) {
  if (n <= 0) return 0;
  if (H <= 0 || dim < 0 || rot < 0 || rank <= 0 || d < rot + rank || ld_q < H * (dim + rot) ||
      (w && ld_down < rank + rot) ||
      ld_out < (H + (w ? 2 : 0)) * d)
    return static_cast<int>(hipErrorInvalidValue);
  int shares = n >= 512 ? 1 : 512 / n;
  if (shares > 8) shares = 8;
  if (shares > H) shares = H;
  if (dtype == 0)
    hipLaunchKernelGGL(latent_split_kernel<float>, dim3(n, shares), dim3(256), 0, s, static_cast<const float*>(q), ld_q,
                       static_cast<const float*>(down), ld_down, static_cast<float*>(qkv), ld_out, w, eps, H, dim, rot, rank, d);
  else if (dtype == 1)
    hipLaunchKernelGGL(latent_split_kernel<bf16_t>, dim3(n, shares), dim3(256), 0, s, static_cast<const bf16_t*>(q), ld_q,
                       static_cast<const bf16_t*>(down), ld_down, static_cast<bf16_t*>(qkv), ld_out, w, eps, H, dim, rot, rank, d);
  else
    return static_cast<int>(hipErrorInvalidValue);
  return kvf_last_error();
}

// out[n, h * out_head + o] = sum_i W[h, o, i] * in[n * ld_in + h * in_head + i]; dtype of rows
// and wtype of W: 0 = fp32, 1 = bf16.  gate (null: none): rows of ld_gate numbers, one per head or (elem) H * O;
// what is stored is the product times sigmoid(gate) times scale.
KVF_EXPORT int kvf_head_product(int dtype, int wtype, const void* in, int ld_in, int in_head, const void* W,
                                void* out, int ld_out, int out_head, int N, int H, int O, int I,
                                const void* gate, int ld_gate, int elem, float scale, hipStream_t s) {
  if (N <= 0) return 0;
  if (H <= 0 || O <= 0 || I <= 0 || H > 65535 || (O + HP_N - 1) / HP_N > 65535 || (gate && N > 1 && ld_gate < (elem ? H * O : H)) ||
      (elem && !gate))
    return static_cast<int>(hipErrorInvalidValue);
  if (dtype == 1 && wtype == 1 && I % 8 == 0 && in_head % 8 == 0 && ld_in % 8 == 0 &&
      reinterpret_cast<uintptr_t>(in) % 16 == 0 && reinterpret_cast<uintptr_t>(W) % 16 == 0) {
    const bf16_t* x = static_cast<const bf16_t*>(in);
    const bf16_t* w = static_cast<const bf16_t*>(W);
    bf16_t* y = static_cast<bf16_t*>(out);
    const HeadGate<bf16_t> g{static_cast<const bf16_t*>(gate), ld_gate, scale};
    const bool wide = ld_out % 4 == 0 && out_head % 4 == 0 && reinterpret_cast<uintptr_t>(out) % 8 == 0;
    return elem ? head_product_mfma_launch<true>(x, ld_in, in_head, w, y, ld_out, out_head, N, H, O, I, wide, g, s)
                : head_product_mfma_launch<false>(x, ld_in, in_head, w, y, ld_out, out_head, N, H, O, I, wide, g, s);
  }
  if (dtype == 0 && wtype == 0)
    return head_product_launch<float, float>(in, ld_in, in_head, W, out, ld_out, out_head, N, H, O, I, gate, ld_gate, elem != 0,
                                              scale, s);
  if (dtype == 1 && wtype == 1)
    return head_product_launch<bf16_t, bf16_t>(in, ld_in, in_head, W, out, ld_out, out_head, N, H, O, I, gate, ld_gate, elem != 0,
                                              scale, s);
  if (dtype == 1 && wtype == 0)
    return head_product_launch<bf16_t, float>(in, ld_in, in_head, W, out, ld_out, out_head, N, H, O, I, gate, ld_gate, elem != 0,
                                              scale, s);
  if (dtype == 0 && wtype == 1)
    return head_product_launch<float, bf16_t>(in, ld_in, in_head, W, out, ld_out, out_head, N, H, O, I, gate, ld_gate, elem != 0,
                                              scale, s);
  return static_cast<int>(hipErrorInvalidValue);
}
