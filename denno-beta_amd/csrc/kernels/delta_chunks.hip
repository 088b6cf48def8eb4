// The delta rule with one decay per row and head, for portions of prompts, on the matrix cores in 32-bit.
//   S <- g S;  e = beta (v - S^T k);  S <- S + k e^T;  o = S^T r          (S [dk, dv] per head, row after row of a request)
// A request's rows are taken 16 at a time.  With S_0 the state before such a chunk, c_t the sum of log g over the chunk's rows up
// to t, and ratio(t, j) = exp(c_t - c_j), the rows of a chunk obey
//   e_t = beta_t (v_t - exp(c_t) S_0^T k_t - sum_{j<t} ratio(t, j) (k_t . k_j) e_j)
// which is (I + M) E = diag(beta) V - diag(beta exp(c)) K S_0 with M strictly lower triangular, so that with X = (I + M)^-1
//   E = U - W S_0,   U = X diag(beta) V,   W = X diag(beta exp(c)) K
//   o_t = exp(c_t) S_0^T r_t + sum_{j<=t} P[t, j] e_j,   P[t, j] = ratio(t, j) (r_t . k_j)
//   S   = exp(c_last) S_0 + sum_t k_t exp(c_last - c_t) e_t^T
// Everything but S_0 is known before the walk: one kernel makes U, W, P, the weighed keys and exp(c) of all chunks side by side,
// a second walks a request's chunks in order, a wave for 16 value columns of a head, the state in its registers.
// All products are v_mfma_f32_16x16x4_f32: operands, sums and state are 32-bit.  Lane l of a wave holds, of an A operand, row
// l % 16 and, in register i of four, column 4 (l / 16) + i of each 16; of a B operand the same of its transpose; of a result, rows
// 4 (l / 16) + i of column l % 16: a result serves as the B operand of the next product as it lies.
#include "common.h"

namespace {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;
constexpr int L = 16;      // rows of a chunk

__device__ __forceinline__ f32x4 mfma(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// The chunks of request s have the numbers from chunk_base(s) on: room for as many as its rows can make.
__device__ __forceinline__ int chunk_base(const int* row_start, int s) { return row_start[s] / L + s; }

struct ChunkArgs {
  const float *r, *k, *v, *zb, *zw, *rate, *bias;
  size_t ldr, ldk, ldv, ldb, ldw;
  float* state;
  size_t slot_stride;
  const int *row_start, *slots;
  int S, H, G, dk, dv, chunks;
  float *U, *W, *P, *KT, *gam;      // per (chunk, head): U [16][dv], W [16][dk], P [16][16], KT [dk][16], gam [16]
  float* out;
  size_t ldo;
};

template <int DB>      // dk / 16
__global__ __launch_bounds__(64) void chunk_parts_kernel(ChunkArgs a) {
  __shared__ float M[L][L + 1], X[L][L + 1], cum[L], bet[L];
  const int id = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, g = lane / 16, n = lane % 16;
  int lo = 0, hi = a.S - 1;      // the last request whose numbers begin at or before id
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (chunk_base(a.row_start, mid) <= id) lo = mid; else hi = mid - 1;
  }
  const int s = lo, row0 = a.row_start[s] + L * (id - chunk_base(a.row_start, s)), rows = min(L, a.row_start[s + 1] - row0);
  if (rows <= 0 || id < chunk_base(a.row_start, s) || a.slots[s] < 0) return;
  constexpr int DK = 16 * DB;
  const int hq = h / (a.H / a.G), dv = a.dv;
  const size_t at = static_cast<size_t>(id) * a.H + h;
  const bool mine = n < rows;
  const size_t row = row0 + (mine ? n : 0);
  f32x4 k[DB], r[DB];
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int b = 0; b < DB; ++b) {
    k[b] = *reinterpret_cast<const f32x4*>(a.k + row * a.ldk + hq * DK + 16 * b + 4 * g);
    r[b] = *reinterpret_cast<const f32x4*>(a.r + row * a.ldr + hq * DK + 16 * b + 4 * g);
    if (!mine) k[b] = zero, r[b] = zero;
  }
  // log g of row n, and its sum over the rows up to n (every group of 16 lanes the same); a row beyond the last: g = 1, beta = 0
  float c = mine ? -a.rate[h] * softplus(a.zw[row * a.ldw + h] + (a.bias ? a.bias[h] : 0.f)) : 0.f;
#pragma unroll
  for (int d = 1; d < L; d *= 2) {
    const float o = __shfl_up(c, d, 16);
    if (n >= d) c += o;
  }
  const float be = mine ? 1.0f / (1.0f + expf(-a.zb[row * a.ldb + h])) : 0.f;
  if (g == 0) cum[n] = c, bet[n] = be;
  f32x4 kk = zero, rk = zero;
#pragma unroll
  for (int b = 0; b < DB; ++b)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      kk = mfma(k[b][i], k[b][i], kk);
      rk = mfma(r[b][i], k[b][i], rk);
    }
  __syncthreads();
  const float last = cum[L - 1];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = 4 * g + i;      // (this lane's result: row t, column n)
    const float ratio = n <= t ? expf(cum[t] - c) : 0.f;
    M[t][n] = n < t ? bet[t] * ratio * kk[i] : 0.f;
    a.P[at * (L * L) + t * L + n] = ratio * rk[i];
  }
  if (g == 0) a.gam[at * L + n] = expf(c);
#pragma unroll
  for (int b = 0; b < DB; ++b)
#pragma unroll
    for (int i = 0; i < 4; ++i) a.KT[(at * DK + 16 * b + 4 * g + i) * L + n] = k[b][i] * expf(last - c);
  __syncthreads();
  // column n of X = (I + M)^-1, row by row (the four groups of lanes do the same work; the first stores)
  float x[L];
#pragma unroll
  for (int t = 0; t < L; ++t) {
    float acc = t == n ? 1.0f : 0.f;
#pragma unroll
    for (int j = 0; j < t; ++j) acc = fmaf(-M[t][j], x[j], acc);
    x[t] = acc;
  }
  if (g == 0) {
#pragma unroll
    for (int t = 0; t < L; ++t) X[t][n] = x[t];
  }
  __syncthreads();
  float xb[4], xg[4];      // X diag(beta) and X diag(beta exp(c)) as A operands: row n, columns 4 g + i
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int j = 4 * g + i;
    xb[i] = X[n][j] * bet[j];
    xg[i] = xb[i] * expf(cum[j]);
  }
  // rows 4 g + i of the chunk, column `col` of a block of 16: the B operand of both products
  size_t src[4];
  bool ok[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) ok[i] = 4 * g + i < rows, src[i] = row0 + (ok[i] ? 4 * g + i : 0);
#pragma unroll
  for (int b = 0; b < DB; ++b) {
    f32x4 w = zero;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float kv = a.k[src[i] * a.ldk + hq * DK + 16 * b + n];
      w = mfma(xg[i], ok[i] ? kv : 0.f, w);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) a.W[at * (L * DK) + (4 * g + i) * DK + 16 * b + n] = w[i];
  }
  for (int c0 = 0; c0 < dv; c0 += 16) {
    const int col = c0 + n;
    f32x4 u = zero;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float vv = a.v[src[i] * a.ldv + static_cast<size_t>(h) * dv + min(col, dv - 1)];
      u = mfma(xb[i], ok[i] ? vv : 0.f, u);
    }
    if (col < dv) {
#pragma unroll
      for (int i = 0; i < 4; ++i) a.U[at * (static_cast<size_t>(L) * dv) + static_cast<size_t>(4 * g + i) * dv + col] = u[i];
    }
  }
}

template <int DB>
__global__ __launch_bounds__(64) void chunk_walk_kernel(ChunkArgs a) {
  constexpr int DK = 16 * DB;
  const int s = blockIdx.z, h = blockIdx.y, lane = threadIdx.x, g = lane / 16, n = lane % 16;
  const int slot = a.slots[s];
  if (slot < 0) return;
  const int row0 = a.row_start[s], row1 = a.row_start[s + 1];
  if (row0 >= row1) return;
  const int hq = h / (a.H / a.G), dv = a.dv;
  const int col = blockIdx.x * 16 + n, cc = min(col, dv - 1);
  const bool live = col < dv;
  const int chunks = (row1 - row0 + L - 1) / L, base = chunk_base(a.row_start, s);
  float* sp = a.state + static_cast<size_t>(slot) * a.slot_stride + (static_cast<size_t>(h) * dv + cc) * DK + 4 * g;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 S[DB];      // S[b][i]: key channel 16 b + 4 g + i of column n
#pragma unroll
  for (int b = 0; b < DB; ++b) {
    // (a head's state may begin at any number of floats)
#pragma unroll
    for (int i = 0; i < 4; ++i) S[b][i] = sp[16 * b + i];
  }
  struct Parts { f32x4 w[DB], r[DB], kt[DB], p, u, gam; float fade; };
  auto fetch = [&](int m) {
    Parts q;
    const size_t at = static_cast<size_t>(base + m) * a.H + h;
    const int t = row0 + L * m + n;
    const float* rr = a.r + static_cast<size_t>(min(t, row1 - 1)) * a.ldr + hq * DK + 4 * g;
#pragma unroll
    for (int b = 0; b < DB; ++b) {
      q.w[b] = *reinterpret_cast<const f32x4*>(a.W + at * (L * DK) + n * DK + 16 * b + 4 * g);
      q.r[b] = *reinterpret_cast<const f32x4*>(rr + 16 * b);
      q.kt[b] = *reinterpret_cast<const f32x4*>(a.KT + (at * DK + 16 * b + n) * L + 4 * g);
    }
    q.p = *reinterpret_cast<const f32x4*>(a.P + at * (L * L) + n * L + 4 * g);
    q.gam = *reinterpret_cast<const f32x4*>(a.gam + at * L + 4 * g);
    q.fade = a.gam[at * L + L - 1];
#pragma unroll
    for (int i = 0; i < 4; ++i) q.u[i] = a.U[at * (static_cast<size_t>(L) * dv) + static_cast<size_t>(4 * g + i) * dv + cc];
    return q;
  };
  Parts now = fetch(0);
  for (int m = 0; m < chunks; ++m) {
    const Parts q = now;
    if (m + 1 < chunks) now = fetch(m + 1);
    // (two sums a product, so that a product does not wait for the one before it)
    f32x4 e0 = zero, e1 = zero, o0 = zero, o1 = zero;
#pragma unroll
    for (int b = 0; b < DB; ++b) {
      e0 = mfma(q.w[b][0], S[b][0], e0);
      o0 = mfma(q.r[b][0], S[b][0], o0);
      e1 = mfma(q.w[b][1], S[b][1], e1);
      o1 = mfma(q.r[b][1], S[b][1], o1);
      e0 = mfma(q.w[b][2], S[b][2], e0);
      o0 = mfma(q.r[b][2], S[b][2], o0);
      e1 = mfma(q.w[b][3], S[b][3], e1);
      o1 = mfma(q.r[b][3], S[b][3], o1);
    }
    f32x4 E, o;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      E[i] = q.u[i] - (e0[i] + e1[i]);
      o[i] = (o0[i] + o1[i]) * q.gam[i];
    }
#pragma unroll
    for (int b = 0; b < DB; ++b) {
#pragma unroll
      for (int i = 0; i < 4; ++i) S[b][i] *= q.fade;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      o = mfma(q.p[i], E[i], o);
#pragma unroll
      for (int b = 0; b < DB; ++b) S[b] = mfma(q.kt[b][i], E[i], S[b]);
    }
    if (live) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = row0 + L * m + 4 * g + i;
        if (t < row1) a.out[static_cast<size_t>(t) * a.ldo + static_cast<size_t>(h) * dv + col] = o[i];
      }
    }
  }
  if (live) {
#pragma unroll
    for (int b = 0; b < DB; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) sp[16 * b + i] = S[b][i];
  }
}

}  // namespace

extern "C" {

// floats of scratch that dn_delta_chunks needs for a step of T rows of S requests
long long dn_delta_chunks_floats(int T, int S, int H, int dk, int dv) {
  return (static_cast<long long>(T) / L + S) * H * (static_cast<long long>(L) * dv + 2LL * L * dk + L * L + L);
}

// r, k [T, G dk], v, out [T, H dv], zb, zw [T, H] (beta = sigmoid(zb), log g = -rate softplus(zw + bias)), 32-bit; dk a multiple of
// 16 up to 128; r and k rows at multiples of 16 bytes; work: dn_delta_chunks_floats floats, at a multiple of 16 bytes
int dn_delta_chunks(const float* r, long long ldr, const float* k, long long ldk, const float* v, long long ldv, const float* zb, long long ldb,
                    const float* zw, long long ldw, const float* rate, const float* bias, float* state, long long slot_stride,
                    const int* row_start, const int* slots, int S, int T, int H, int G, int dk, int dv, float* work, float* out,
                    long long ldo, hipStream_t stream) {
  auto by16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (dk < 16 || dk > 128 || dk % 16 != 0 || dv < 1 || H < 1 || G < 1 || H % G != 0 || S < 1 || S > 65535 || H > 65535 || !rate || ldr % 4 != 0 ||
      ldk % 4 != 0 || !by16(r) || !by16(k) || !by16(work) || slot_stride < static_cast<long long>(H) * dk * dv)
    return DN_ERR_SHAPE;
  if (T == 0) return 0;
  const int chunks = T / L + S;
  const size_t n = static_cast<size_t>(chunks) * H;
  // (pieces whose lengths are multiples of 16 floats first, so that each begins at a multiple of 16 bytes)
  float* W = work;
  float* KT = W + n * L * dk;
  float* P = KT + n * L * dk;
  float* gam = P + n * L * L;
  float* U = gam + n * L;
  const ChunkArgs a{r, k, v, zb, zw, rate, bias, static_cast<size_t>(ldr), static_cast<size_t>(ldk), static_cast<size_t>(ldv), static_cast<size_t>(ldb),
                    static_cast<size_t>(ldw), state, static_cast<size_t>(slot_stride), row_start, slots, S, H, G, dk, dv, chunks, U, W, P, KT, gam, out,
                    static_cast<size_t>(ldo)};
#define DN_CHUNKS(DB)                                                                                                            \
  case 16 * DB:                                                                                                                  \
    hipLaunchKernelGGL(chunk_parts_kernel<DB>, dim3(chunks, H), dim3(64), 0, stream, a);                                          \
    hipLaunchKernelGGL(chunk_walk_kernel<DB>, dim3((dv + 15) / 16, H, S), dim3(64), 0, stream, a);                                \
    break
  switch (dk) {
    DN_CHUNKS(1);
    DN_CHUNKS(2);
    DN_CHUNKS(3);
    DN_CHUNKS(4);
    DN_CHUNKS(5);
    DN_CHUNKS(6);
    DN_CHUNKS(7);
    DN_CHUNKS(8);
    default: return DN_ERR_SHAPE;
  }
#undef DN_CHUNKS
  return dn_launch_status();
}

}  // extern "C"
