// Linear attention with one scalar decay per head and token over packed batches (see seqmix.hip for
// the layout of chunks, positions and state slots), in two designs that share every kernel:
//
//   constant decay    S <- decay[h] S + k v^T,  o = S^T q         q, k, v through silu
//   matrix memory     a = cap tanh((zi + bi) / cap),  b = log sigmoid(cap tanh((zf + bf) / cap))
//                     m' = max(b + m, a);  S <- e^(b + m - m') S + e^(a - m') k v^T;  n the same sum over the keys
//                     o = S^T q / (max(|n . q|, e^-m') + 1e-6)         q times a constant
//
// State, per slot and head: S [d, dv], then (matrix memory) n [d], padded to a multiple of 4 floats;
// the running maximum m is a separate [slots, heads].  A chunk that starts at position 0 starts from zeros.
//
// Steps that hold portions of prompts go by tiles of up to C rows of a chunk (the tile list comes from
// the host).  With F_t the log decay summed from the tile's first row to row t, unrolling the
// recurrence over a tile gives
//   S_end = e^(F_end + m_start - m_end) S_start + sum_j e^(F_end - F_j + a_j - m_end) k_j v_j^T
//   o_i ~ e^(F_i + m_start - m_i) S_start^T q_i + sum_{j <= i} e^(F_i - F_j + a_j - m_i) (q_i . k_j) v_j
// (m and a are zero for the constant decay; every exponent is <= 0 by the definition of m), so that
//   1  mlstm_gates        a, F and m of every row: a (+, max) scan per sequence and head
//   2  la_states          every tile's sum_j, all tiles at once                      -> workspace
//   3  la_scan            the states at the tiles' starts, walked tile by tile (elementwise) -> workspace, state
//   4  la_out             every tile's outputs, all tiles at once
// 2 and 4 are matrix products and run on the matrix cores in fp32 (16x16x4): the state and all that
// enters the recurrence stay 32-bit whatever the storage type.  F is summed and subtracted in double.
// Steps of a few tokens per sequence (decode) take la_step: one workgroup per (sequence, head) reads the
// state once, updates it in place and finishes the head (matrix memory: also its gates, norm and output
// gate).
#include "common.h"

namespace mi355 {

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float log_sigmoid_f(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

struct LaDims {
  int H, d, dv;
  int us;                       // floats of one head's state: d * dv (+ d), padded to a multiple of 4
  int C;                        // rows of a tile
};

// rows [0, n) x cols [0, d) of a row-strided tensor -> fp32 LDS [rows_p][ld], activation and a factor per
// row applied, zeros up to rows_p rows and cols_p columns
template <typename T>
__device__ __forceinline__ void stage_rows(float* dst, int ld, const typename Elem<T>::S* base, const typename Elem<T>::S* src,
                                           int64_t stride, int n, int rows_p, int d, int cols_p, int silu, float scale,
                                           const float* row_factor, int vec) {
  if constexpr (sizeof(typename Elem<T>::S) == 2) {
    if (vec) {                                           // d a multiple of 8, rows on 16-byte boundaries
      const int per = cols_p >> 3;
      for (int i = threadIdx.x; i < rows_p * per; i += blockDim.x) {
        const int r = i / per, c = (i - r * per) * 8;
        float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (r < n && c < d) {
          unpack8<T>(MI355_LD(uint4, base, src + r * stride + c), f);
          const float w = row_factor != nullptr ? row_factor[r] : 1.0f;
#pragma unroll
          for (int j = 0; j < 8; ++j) f[j] = (silu ? silu_f(f[j]) : f[j] * scale) * w;
        }
        float4* o = reinterpret_cast<float4*>(dst + r * ld + c);
        o[0] = make_float4(f[0], f[1], f[2], f[3]);
        o[1] = make_float4(f[4], f[5], f[6], f[7]);
      }
      return;
    }
  }
  for (int i = threadIdx.x; i < rows_p * cols_p; i += blockDim.x) {
    const int r = i / cols_p, c = i - r * cols_p;
    float f = 0.f;
    if (r < n && c < d) {
      f = MI355_LDF(T, base, src + r * stride + c);
      f = (silu ? silu_f(f) : f * scale) * (row_factor != nullptr ? row_factor[r] : 1.0f);
    }
    dst[r * ld + c] = f;
  }
}

// ---- 1: a, F, m of every row.  One workgroup per (chunk, head): its 16 waves scan a tile each (lane = row), then
// m at the tiles' starts follows from the tiles' ends, wave by wave.  ga / gm [H][T] float, gf [H][T] double,
// mstart [tiles][H].
__global__ __launch_bounds__(1024) void mlstm_gates_kernel(float* __restrict__ ga, double* __restrict__ gf, float* __restrict__ gm,
                                                           float* __restrict__ mstart, const float* __restrict__ z,
                                                           const float* __restrict__ bias, float cap, float* __restrict__ m_state,
                                                           const int32_t* __restrict__ cu_seqlens,
                                                           const int64_t* __restrict__ positions,
                                                           const int32_t* __restrict__ state_slots,
                                                           const int32_t* __restrict__ tile_start, int H, int C, int64_t T) {
  constexpr int NW = 16;
  __shared__ double ends[2][NW];                          // F and M of the tiles' last rows
  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t cs = MI355_LD(int32_t, cu_seqlens, cu_seqlens + s);
  const int64_t n = MI355_LD(int32_t, cu_seqlens, cu_seqlens + s + 1) - cs;
  if (n <= 0) return;                                     // (the whole workgroup)
  const int64_t slot = MI355_LD(int32_t, state_slots, state_slots + s);
  const int64_t tile0 = MI355_LD(int32_t, tile_start, tile_start + s);
  float m0 = MI355_LD(int64_t, positions, positions + cs) == 0 ? 0.f : MI355_LD(float, m_state, m_state + slot * H + h);
  const float bi = MI355_LD(float, bias, bias + h), bf = MI355_LD(float, bias, bias + H + h);
  const int64_t num = (n + C - 1) / C;
  for (int64_t g = 0; g < num; g += NW) {
    const int64_t r0 = (g + wave) * C;
    const bool live = lane < C && r0 + lane < n;
    const int64_t t = cs + r0 + lane;
    float a = 0.f;
    double F = 0.0, M = -1.0e300;
    if (live) {
      a = cap * tanhf((MI355_LD(float, z, z + t * 2 * H + h) + bi) / cap);
      F = log_sigmoid_f(cap * tanhf((MI355_LD(float, z, z + t * 2 * H + H + h) + bf) / cap));
      M = a;
    }
    // (F, M) of rows up to this one: (F1, M1) then (F2, M2) is (F1 + F2, max(M1 + F2, M2))
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double Fp = __shfl_up(F, o, 64), Mp = __shfl_up(M, o, 64);
      if (lane >= o) {
        M = fmax(Mp + F, M);
        F += Fp;
      }
    }
    if (lane == 63) ends[0][wave] = F, ends[1][wave] = M; // (rows past the tile's last add nothing to either)
    __syncthreads();
    float mine = m0;                                      // m ahead of this wave's tile
    for (int w = 0; w < NW; ++w) {
      if (w == wave) mine = m0;
      m0 = static_cast<float>(fmax(ends[1][w], ends[0][w] + static_cast<double>(m0)));
    }
    if (live) {
      MI355_ST(float, ga, ga + h * T + t, a);
      MI355_ST(double, gf, gf + h * T + t, F);
      MI355_ST(float, gm, gm + h * T + t, static_cast<float>(fmax(M, F + static_cast<double>(mine))));
    }
    if (lane == 0 && g + wave < num) MI355_ST(float, mstart, mstart + (tile0 + g + wave) * H + h, mine);
    __syncthreads();                                      // the ends are read before the next turn writes them
  }
  if (threadIdx.x == 0) MI355_ST(float, m_state, m_state + slot * H + h, m0);
}

// ---- 2: sum_j e^(F_end - F_j + a_j - m_end) k_j v_j^T of every tile and head
template <typename T, bool MEM>
__global__ __launch_bounds__(256) void la_states_kernel(
    float* __restrict__ ws, const typename Elem<T>::S* __restrict__ k, int64_t k_stride,
    const typename Elem<T>::S* __restrict__ v, int64_t v_stride, const double* __restrict__ log_decay,
    const float* __restrict__ ga, const double* __restrict__ gf, const float* __restrict__ gm,
    const float* __restrict__ mstart, const int32_t* __restrict__ tiles, LaDims D, int64_t total_rows, int64_t num_tiles,
    int vec) {
  extern __shared__ float lds[];
  const int tile = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int d = D.d, dv = D.dv, dp = (d + 15) & ~15, dvp = (dv + 15) & ~15;
  const int kl = ((dp + 63) & ~63) + 16, vl = ((dvp + 63) & ~63) + 16;      // row strides: four rows on four sixteenths of the banks
  float* Ks = lds;
  float* Vs = Ks + D.C * kl;
  float* wr = Vs + D.C * vl;
  const int64_t row0 = MI355_LD(int32_t, tiles, tiles + 3 * tile + 1);
  const int n = MI355_LD(int32_t, tiles, tiles + 3 * tile + 2);
  const int np = (n + 3) & ~3;
  for (int i = tid; i < n; i += blockDim.x) {
    if (MEM) {
      const int64_t at = h * total_rows + row0;
      const double e = MI355_LD(double, gf, gf + at + n - 1) - MI355_LD(double, gf, gf + at + i) +
                       static_cast<double>(MI355_LD(float, ga, ga + at + i)) -
                       static_cast<double>(MI355_LD(float, gm, gm + at + n - 1));
      wr[i] = expf(static_cast<float>(e));
    } else {
      wr[i] = expf(static_cast<float>((n - 1 - i) * MI355_LD(double, log_decay, log_decay + h)));
    }
  }
  if (tid == 0) {                                         // the factor on the tile's incoming state, for la_scan
    float f;
    if (MEM) {
      const int64_t end = h * total_rows + row0 + n - 1;
      f = expf(static_cast<float>(MI355_LD(double, gf, gf + end) +
                                  static_cast<double>(MI355_LD(float, mstart, mstart + static_cast<int64_t>(tile) * D.H + h)) -
                                  static_cast<double>(MI355_LD(float, gm, gm + end))));
    } else {
      f = expf(static_cast<float>(n * MI355_LD(double, log_decay, log_decay + h)));
    }
    MI355_ST(float, ws, ws + num_tiles * D.H * D.us + static_cast<int64_t>(tile) * D.H + h, f);
  }
  __syncthreads();
  stage_rows<T>(Ks, kl, k, k + row0 * k_stride + static_cast<int64_t>(h) * d, k_stride, n, np, d, dp, !MEM, 1.0f, wr, vec);
  stage_rows<T>(Vs, vl, v, v + row0 * v_stride + static_cast<int64_t>(h) * dv, v_stride, n, np, dv, dvp, !MEM, 1.0f, nullptr, vec);
  __syncthreads();
  float* U = ws + (static_cast<int64_t>(tile) * D.H + h) * D.us;
  const int wave = tid >> 6, lane = tid & 63, li = lane & 15, kk = lane >> 4;
  const int mt = dp >> 4, nt = dvp >> 4, mb = (mt + 1) >> 1, nb = (nt + 1) >> 1;
  for (int blk = wave; blk < mb * nb; blk += static_cast<int>(blockDim.x >> 6)) {
    const int m0 = (blk / nb) * 2, n0 = (blk % nb) * 2;
    const bool m1 = m0 + 1 < mt, n1 = n0 + 1 < nt;
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float* ka = Ks + kk * kl + m0 * 16 + li;
    const float* vb = Vs + kk * vl + n0 * 16 + li;
    for (int r = 0; r < np; r += 4) {
      const float a0 = ka[r * kl], a1 = m1 ? ka[r * kl + 16] : 0.f;
      const float b0 = vb[r * vl], b1 = n1 ? vb[r * vl + 16] : 0.f;
      acc[0][0] = mfma_f32(a0, b0, acc[0][0]);
      acc[0][1] = mfma_f32(a0, b1, acc[0][1]);
      acc[1][0] = mfma_f32(a1, b0, acc[1][0]);
      acc[1][1] = mfma_f32(a1, b1, acc[1][1]);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = (m0 + i) * 16 + 4 * kk + r, col = (n0 + j) * 16 + li;
          if (row < d && col < dv) MI355_ST(float, ws, U + static_cast<int64_t>(row) * dv + col, acc[i][j][r]);
        }
  }
  for (int c = d * dv + tid; c < D.us; c += blockDim.x) {    // n, and the padding
    float sum = 0.f;
    const int i = c - d * dv;
    if (MEM && i < d)
      for (int r = 0; r < n; ++r) sum += Ks[r * kl + i];
    MI355_ST(float, ws, U + c, sum);
  }
}

// ---- 3: tile by tile, elementwise: ws[tile] becomes the state at the tile's start
__global__ __launch_bounds__(256) void la_scan_kernel(float* __restrict__ ws, float* __restrict__ state,
                                                      const int32_t* __restrict__ cu_seqlens,
                                                      const int64_t* __restrict__ positions,
                                                      const int32_t* __restrict__ state_slots,
                                                      const int32_t* __restrict__ tile_start, LaDims D, int64_t num_tiles) {
  const int h = blockIdx.y, s = blockIdx.z;
  const int t0 = MI355_LD(int32_t, tile_start, tile_start + s), t1 = MI355_LD(int32_t, tile_start, tile_start + s + 1);
  if (t0 >= t1) return;
  const int e4 = blockIdx.x * blockDim.x + threadIdx.x;
  if (4 * e4 >= D.us) return;
  const int64_t slot = MI355_LD(int32_t, state_slots, state_slots + s);
  const int64_t cs = MI355_LD(int32_t, cu_seqlens, cu_seqlens + s);
  float* sp = state + (slot * D.H + h) * D.us + 4 * e4;
  float4 S = make_float4(0.f, 0.f, 0.f, 0.f);
  if (MI355_LD(int64_t, positions, positions + cs) != 0) S = MI355_LD(float4, state, sp);
  const int64_t step = static_cast<int64_t>(D.H) * D.us;
  float* w = ws + (static_cast<int64_t>(t0) * D.H + h) * D.us + 4 * e4;
  const float* fac = ws + num_tiles * step + static_cast<int64_t>(t0) * D.H + h;
  constexpr int PF = 8;
  for (int t = 0; t < t1 - t0; t += PF) {
    float4 u[PF];
    float f[PF];
#pragma unroll
    for (int j = 0; j < PF; ++j) {
      u[j] = make_float4(0.f, 0.f, 0.f, 0.f);
      f[j] = 1.f;
      if (t + j < t1 - t0) {
        u[j] = MI355_LD(float4, ws, w + (t + j) * step);
        f[j] = MI355_LD(float, ws, fac + static_cast<int64_t>(t + j) * D.H);
      }
    }
#pragma unroll
    for (int j = 0; j < PF; ++j) {
      if (t + j < t1 - t0) {
        MI355_ST(float4, ws, w + (t + j) * step, S);
        S.x = f[j] * S.x + u[j].x, S.y = f[j] * S.y + u[j].y, S.z = f[j] * S.z + u[j].z, S.w = f[j] * S.w + u[j].w;
      }
    }
  }
  MI355_ST(float4, state, sp, S);
}

// ---- 4: outputs of every tile and head, fp32 [T][H][dv]
template <typename T, bool MEM>
__global__ __launch_bounds__(512) void la_out_kernel(
    float* __restrict__ o, const float* __restrict__ ws, const typename Elem<T>::S* __restrict__ q, int64_t q_stride,
    const typename Elem<T>::S* __restrict__ k, int64_t k_stride, const typename Elem<T>::S* __restrict__ v, int64_t v_stride,
    float q_scale, const double* __restrict__ log_decay, const float* __restrict__ ga, const double* __restrict__ gf,
    const float* __restrict__ gm, const float* __restrict__ mstart, const int32_t* __restrict__ tiles, LaDims D,
    int64_t total_rows, int vec) {
  extern __shared__ float lds[];
  const int tile = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int d = D.d, dv = D.dv, dp = (d + 15) & ~15, dvp = (dv + 15) & ~15, C = D.C;
  const int ql = ((dp + 63) & ~63) + 4, vl = ((dvp + 63) & ~63) + 16, pl = 68;
  float* Qs = lds;
  float* Ks = Qs + C * ql;
  float* Vs = Ks + C * ql;
  float* Ps = Vs + C * vl;
  double* Fr = reinterpret_cast<double*>(Ps + C * pl);          // (C * pl floats: a multiple of two)
  float* ar = reinterpret_cast<float*>(Fr + C);                 // a_j
  float* mr = ar + C;                                           // m_i
  float* er = mr + C;                                           // e^(F_i + m_start - m_i)
  float* dr = er + C;                                           // 1 / denominator
  const int64_t row0 = MI355_LD(int32_t, tiles, tiles + 3 * tile + 1);
  const int n = MI355_LD(int32_t, tiles, tiles + 3 * tile + 2);
  const int np = (n + 15) & ~15;
  for (int i = tid; i < np; i += blockDim.x) {
    double F = 0.0;
    float a = 0.f, m = 0.f, e = 0.f;
    if (i < n) {
      double m0 = 0.0;
      if (MEM) {
        const int64_t at = h * total_rows + row0 + i;
        F = MI355_LD(double, gf, gf + at);
        a = MI355_LD(float, ga, ga + at);
        m = MI355_LD(float, gm, gm + at);
        m0 = MI355_LD(float, mstart, mstart + static_cast<int64_t>(tile) * D.H + h);
      } else {
        F = (i + 1) * MI355_LD(double, log_decay, log_decay + h);
      }
      e = expf(static_cast<float>(F + m0 - static_cast<double>(m)));
    }
    Fr[i] = F, ar[i] = a, mr[i] = m, er[i] = e;
  }
  stage_rows<T>(Qs, ql, q, q + row0 * q_stride + static_cast<int64_t>(h) * d, q_stride, n, np, d, dp, !MEM, q_scale, nullptr, vec);
  stage_rows<T>(Ks, ql, k, k + row0 * k_stride + static_cast<int64_t>(h) * d, k_stride, n, np, d, dp, !MEM, 1.0f, nullptr, vec);
  stage_rows<T>(Vs, vl, v, v + row0 * v_stride + static_cast<int64_t>(h) * dv, v_stride, n, np, dv, dvp, !MEM, 1.0f, nullptr, vec);
  __syncthreads();
  const int wave = tid >> 6, lane = tid & 63, li = lane & 15, kk = lane >> 4, nw = blockDim.x >> 6;
  const int rb = np >> 4;
  // P = Q K^T under the decay weights, blocks on and below the diagonal
  for (int blk = wave; blk < rb * (rb + 1) / 2; blk += nw) {
    int bi = 0, bj = blk;
    while (bj > bi) bj -= ++bi;                          // blk = bi (bi + 1) / 2 + bj
    f32x4 p0 = f32x4{0.f, 0.f, 0.f, 0.f}, p1 = p0;
    const float* qa = Qs + (bi * 16 + li) * ql + kk;
    const float* kb = Ks + (bj * 16 + li) * ql + kk;
    for (int c = 0; c < dp; c += 8) {
      p0 = mfma_f32(qa[c], kb[c], p0);
      p1 = mfma_f32(qa[c + 4], kb[c + 4], p1);
    }
    const int j = bj * 16 + li;
    const double Fj = Fr[j];
    const double aj = ar[j];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = bi * 16 + 4 * kk + r;
      float w = 0.f;
      if (j <= i && i < n) {
        // the constant decay by the row distance, so that a decay of zero (log: a huge negative number) keeps its diagonal
        const double ex = MEM ? Fr[i] - Fj + aj - static_cast<double>(mr[i])
                              : (i - j) * MI355_LD(double, log_decay, log_decay + h);
        w = expf(static_cast<float>(ex)) * (p0[r] + p1[r]);
      }
      Ps[i * pl + j] = w;
    }
  }
  const float* S = ws + (static_cast<int64_t>(tile) * D.H + h) * D.us;
  __syncthreads();
  if (MEM) {
    for (int c = tid; c < d; c += blockDim.x) Ks[c] = MI355_LD(float, ws, S + static_cast<int64_t>(d) * dv + c);
    __syncthreads();
  }
  if (MEM) {
    // n . q: the rows' sums of P, and the state's part; 8 adjacent lanes per row (n lies over the keys, which are done with)
    for (int i = tid >> 3; i < np; i += blockDim.x >> 3) {
      const int u = tid & 7;
      float sum = 0.f, nq = 0.f;
      for (int j = u; j < np && j <= i; j += 8) sum += Ps[i * pl + j];
      for (int c = u; c < d; c += 8) nq += Ks[c] * Qs[i * ql + c];
      sum += er[i] * nq;
      sum += __shfl_xor(sum, 1, 64);
      sum += __shfl_xor(sum, 2, 64);
      sum += __shfl_xor(sum, 4, 64);
      if (u == 0) dr[i] = 1.0f / (fmaxf(fabsf(sum), expf(-mr[i])) + 1e-6f);
    }
    __syncthreads();
  }
  const int nt = dvp >> 4, nb = (nt + 3) >> 2;
  for (int blk = wave; blk < rb * nb; blk += nw) {
    const int bi = blk / nb, n0 = (blk % nb) * 4;
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float* qa = Qs + (bi * 16 + li) * ql + kk;
    // the incoming state's part: 16 rows of it at a time, the next 16 on their way meanwhile.  Rows and columns past
    // the head read its last ones: the former meet zeros of Q, the latter are not stored.
    const float* sc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int col = (n0 + j) * 16 + li;
      sc[j] = S + (col < dv ? col : dv - 1);
    }
    float b[4][4], bn[4][4];
    auto fetch = [&](float (&x)[4][4], int c) {
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int row = c + 4 * u + kk;
        const int64_t at = static_cast<int64_t>(row < d ? row : d - 1) * dv;
#pragma unroll
        for (int j = 0; j < 4; ++j) x[u][j] = MI355_LD(float, ws, sc[j] + at);
      }
    };
    auto work = [&](const float (&x)[4][4], int c) {
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float a = qa[c + 4 * u];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = mfma_f32(a, x[u][j], acc[j]);
      }
    };
    fetch(b, 0);
    for (int c = 0; c < dp; c += 32) {
      if (c + 16 < dp) fetch(bn, c + 16);
      work(b, c);
      if (c + 16 >= dp) break;
      if (c + 32 < dp) fetch(b, c + 32);
      work(bn, c + 16);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[j][r] *= er[bi * 16 + 4 * kk + r];
    const float* pa = Ps + (bi * 16 + li) * pl + kk;
    const float* vb = Vs + kk * vl + n0 * 16 + li;
    for (int c = 0; c < bi * 16 + 16; c += 4) {
      const float a = pa[c];
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[j] = mfma_f32(a, n0 + j < nt ? vb[c * vl + 16 * j] : 0.f, acc[j]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = bi * 16 + 4 * kk + r;
      if (i >= n) continue;
      const float f = MEM ? dr[i] : 1.0f;
      float* op = o + ((row0 + i) * D.H + h) * dv;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int col = (n0 + j) * 16 + li;
        if (col < dv) MI355_ST(float, o, op + col, acc[j][r] * f);
      }
    }
  }
}

// ---- chunks of a few tokens: one workgroup per (chunk, head), the state updated in place
struct LaStepMem {                // matrix memory only: what its gates, norm and output gate read
  const float* x;                 // fp32 rows the gate projections read
  int64_t x_stride;
  const void* gate_w;             // [2 H, width]: input gates, then forget gates
  const float* gate_b;            // [2 H]
  int width;
  float cap;
  float* m_state;                 // [slots, H]
  const void* g;                  // output gate rows [T, H dv]
  int64_t g_stride;
  const float* norm;              // [H dv]
  float eps;
  void* out;                      // [T, H dv] in the storage type
  int64_t out_stride;
};

template <typename T, bool MEM, int VW>
__global__ __launch_bounds__(256) void la_step_kernel(
    float* __restrict__ o, const typename Elem<T>::S* __restrict__ q, int64_t q_stride,
    const typename Elem<T>::S* __restrict__ k, int64_t k_stride, const typename Elem<T>::S* __restrict__ v, int64_t v_stride,
    float q_scale, const double* __restrict__ log_decay, float* __restrict__ state, const int32_t* __restrict__ cu_seqlens,
    const int64_t* __restrict__ positions, const int32_t* __restrict__ state_slots, LaDims D, LaStepMem M) {
  typedef typename Elem<T>::S E;
  extern __shared__ float lds[];
  __shared__ float scratch[32];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int d = D.d, dv = D.dv;
  const int nc = dv / VW;                                 // columns of VW floats
  const int cg = nc < 256 ? nc : 256;                     // columns worked on at a time
  const int rg = 256 / cg;                                // row groups beside each other
  float* qs = lds;                                        // [d]
  float* ks = qs + d;                                     // [d]
  float* ob = ks + d;                                     // [dv] the head's output
  float* part = ob + dv;                                  // [rg][cg * VW]
  const int64_t cs = MI355_LD(int32_t, cu_seqlens, cu_seqlens + s);
  const int64_t n = MI355_LD(int32_t, cu_seqlens, cu_seqlens + s + 1) - cs;
  if (n <= 0) return;
  const int64_t slot = MI355_LD(int32_t, state_slots, state_slots + s);
  float* sp = state + (slot * D.H + h) * D.us;
  bool fresh = MI355_LD(int64_t, positions, positions + cs) == 0;
  float m = 0.f;
  if (MEM && !fresh) m = MI355_LD(float, M.m_state, M.m_state + slot * D.H + h);
  const float dec = MEM ? 0.f : expf(static_cast<float>(MI355_LD(double, log_decay, log_decay + h)));
  const int tx = tid % cg, ty = tid / cg;
  constexpr int PF = 8;
  float S[PF][VW];
  // rows i0, i0 + rg, ... of column group c of the state
  auto fetch = [&](int i0, int c) {
#pragma unroll
    for (int u = 0; u < PF; ++u) {
      const int i = i0 + u * rg;
      if constexpr (VW == 4) {
        float4 x4 = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i < d && !fresh) x4 = MI355_LD(float4, state, sp + static_cast<int64_t>(i) * dv + c * 4);
        S[u][0] = x4.x, S[u][1] = x4.y, S[u][2] = x4.z, S[u][3] = x4.w;
      } else {
        S[u][0] = i < d && !fresh ? MI355_LD(float, state, sp + static_cast<int64_t>(i) * dv + c) : 0.f;
      }
    }
  };
  for (int64_t t = cs; t < cs + n; ++t) {
    __syncthreads();                                      // the previous token's reads of LDS are done
    if (ty < rg) fetch(ty, tx);                           // the first rows travel while the gates are worked out
    for (int i = tid; i < d; i += 256) {
      const float qv = MI355_LDF(T, q, q + t * q_stride + static_cast<int64_t>(h) * d + i);
      const float kv = MI355_LDF(T, k, k + t * k_stride + static_cast<int64_t>(h) * d + i);
      qs[i] = MEM ? qv * q_scale : silu_f(qv);
      ks[i] = MEM ? kv : silu_f(kv);
    }
    float r = dec, w = 1.0f;
    if (MEM) {
      const E* wi = static_cast<const E*>(M.gate_w) + static_cast<int64_t>(h) * M.width;
      const E* wf = wi + static_cast<int64_t>(D.H) * M.width;
      float zi = 0.f, zf = 0.f;
      for (int i = tid; i < M.width; i += 256) {
        const float xv = MI355_LD(float, M.x, M.x + t * M.x_stride + i);
        zi += xv * MI355_LDF(T, M.gate_w, wi + i);
        zf += xv * MI355_LDF(T, M.gate_w, wf + i);
      }
      zi = block_sum32(zi, scratch) + MI355_LD(float, M.gate_b, M.gate_b + h);
      zf = block_sum32(zf, scratch) + MI355_LD(float, M.gate_b, M.gate_b + D.H + h);
      const float a = M.cap * tanhf(zi / M.cap), b = log_sigmoid_f(M.cap * tanhf(zf / M.cap));
      const float m2 = fmaxf(b + m, a);
      r = expf(b + m - m2);
      w = expf(a - m2);
      m = m2;
    }
    if (fresh) r = 0.f;
    __syncthreads();
    float den = 1.0f;
    if (MEM) {
      float nq = 0.f;
      for (int i = tid; i < d; i += 256) {
        float* np = sp + static_cast<int64_t>(d) * dv + i;
        const float nv = (fresh ? 0.f : r * MI355_LD(float, state, np)) + w * ks[i];
        MI355_ST(float, state, np, nv);
        nq += nv * qs[i];
      }
      den = 1.0f / (fmaxf(fabsf(block_sum32(nq, scratch)), expf(-m)) + 1e-6f);
    }
    for (int c0 = 0; c0 < nc; c0 += cg) {                 // (one turn for up to 256 columns of VW)
      const int c = c0 + tx;
      const bool live = ty < rg && c < nc;
      float vv[VW], acc[VW];
#pragma unroll
      for (int j = 0; j < VW; ++j) {
        acc[j] = 0.f;
        vv[j] = 0.f;
        if (live) {
          vv[j] = MI355_LDF(T, v, v + t * v_stride + static_cast<int64_t>(h) * dv + c * VW + j);
          if (!MEM) vv[j] = silu_f(vv[j]);
          vv[j] *= w;
        }
      }
      if (live) {
        for (int i0 = ty; i0 < d; i0 += PF * rg) {
          if (c0 > 0 || i0 > ty) fetch(i0, c);
#pragma unroll
          for (int u = 0; u < PF; ++u) {
            const int i = i0 + u * rg;
            if (i >= d) continue;
            const float kv = ks[i], qv = qs[i];
#pragma unroll
            for (int j = 0; j < VW; ++j) {
              S[u][j] = r * S[u][j] + kv * vv[j];
              acc[j] += S[u][j] * qv;
            }
            if constexpr (VW == 4)
              MI355_ST(float4, state, sp + static_cast<int64_t>(i) * dv + c * 4, make_float4(S[u][0], S[u][1], S[u][2], S[u][3]));
            else
              MI355_ST(float, state, sp + static_cast<int64_t>(i) * dv + c, S[u][0]);
          }
        }
#pragma unroll
        for (int j = 0; j < VW; ++j) part[ty * cg * VW + tx * VW + j] = acc[j];
      }
      __syncthreads();
      for (int i = tid; i < cg * VW; i += 256) {
        if (c0 * VW + i >= dv) continue;
        float sum = 0.f;
        for (int g = 0; g < rg; ++g) sum += part[g * cg * VW + i];
        ob[c0 * VW + i] = sum * den;
      }
      __syncthreads();
    }
    if (MEM) {
      float ss = 0.f;
      for (int i = tid; i < dv; i += 256) ss += ob[i] * ob[i];
      const float rn = 1.0f / sqrtf(block_sum32(ss, scratch) / static_cast<float>(dv) + M.eps);
      for (int i = tid; i < dv; i += 256) {
        const int64_t hc = static_cast<int64_t>(h) * dv + i;
        const float g = MI355_LDF(T, M.g, static_cast<const E*>(M.g) + t * M.g_stride + hc);
        MI355_STF(T, M.out, static_cast<E*>(M.out) + t * M.out_stride + hc,
                  ob[i] * rn * MI355_LD(float, M.norm, M.norm + hc) / (1.0f + expf(-g)));
      }
    } else {
      for (int i = tid; i < dv; i += 256) MI355_ST(float, o, o + (t * D.H + h) * dv + i, ob[i]);
    }
    fresh = false;
  }
  if (MEM && tid == 0) MI355_ST(float, M.m_state, M.m_state + slot * D.H + h, m);
}

static inline int64_t la_state_floats(int d, int dv, bool mem) { return (static_cast<int64_t>(d) * dv + (mem ? d : 0) + 3) / 4 * 4; }

static inline int64_t la_states_lds(int C, int d, int dv) {
  const int dp = (d + 15) & ~15, dvp = (dv + 15) & ~15;
  return sizeof(float) * (static_cast<int64_t>(C) * (((dp + 63) & ~63) + 16 + ((dvp + 63) & ~63) + 16) + C);
}
static inline int64_t la_out_lds(int C, int d, int dv) {
  const int dp = (d + 15) & ~15, dvp = (dv + 15) & ~15;
  return sizeof(float) * (static_cast<int64_t>(C) * (2 * (((dp + 63) & ~63) + 4) + ((dvp + 63) & ~63) + 16 + 68) + 6 * C);
}
constexpr int64_t kLdsBytes = 160 * 1024;

}  // namespace mi355

using namespace mi355;

#define REQ_DTYPE(dtype) MI355_REQUIRE((dtype) >= MI355_BF16 && (dtype) <= MI355_F32, MI355_ERR_UNSUPPORTED, "dtype code %d", (dtype))

extern "C" int64_t mi355_linear_attn_state_floats(int32_t head_dim, int32_t v_dim, int32_t normalizer) {
  return la_state_floats(head_dim, v_dim, normalizer != 0);
}

// rows of a tile: as many (64, 32, 16) as the workgroup's LDS holds; 0: the sizes do not fit
extern "C" int32_t mi355_linear_attn_tile_rows(int32_t head_dim, int32_t v_dim) {
  for (int c = 64; c >= 16; c >>= 1)
    if (la_out_lds(c, head_dim, v_dim) <= kLdsBytes && la_states_lds(c, head_dim, v_dim) <= kLdsBytes) return c;
  return 0;
}

extern "C" int32_t mi355_mlstm_gates(float* log_in, double* log_decay_sum, float* running_max, float* tile_max, const float* z,
                                     const float* bias, float cap, float* m_state, const int32_t* cu_seqlens,
                                     const int64_t* positions, const int32_t* state_slots, const int32_t* tile_start,
                                     int32_t num_seqs, int32_t num_heads, int32_t tile_rows, int64_t num_tokens,
                                     void* stream) {
  MI355_REQUIRE(log_in && log_decay_sum && running_max && tile_max && z && bias && m_state && cu_seqlens && positions &&
                    state_slots && tile_start,
                MI355_ERR_INVALID, "mlstm_gates: null pointer");
  MI355_REQUIRE(num_seqs >= 0 && num_heads > 0 && num_heads <= 65535 && tile_rows > 0 && tile_rows <= 64 && num_tokens >= 0 && cap > 0.f,
                MI355_ERR_INVALID, "mlstm_gates: sizes");
  if (num_seqs == 0 || num_tokens == 0) return MI355_OK;
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(num_seqs, num_heads), dim3(1024), 0, static_cast<hipStream_t>(stream), log_in,
                     log_decay_sum, running_max, tile_max, z, bias, cap, m_state, cu_seqlens, positions, state_slots,
                     tile_start, num_heads, tile_rows, num_tokens);
  return check_launch("mlstm_gates");
}

extern "C" int32_t mi355_linear_attn_chunks(float* o, const void* q, int64_t q_stride, const void* k, int64_t k_stride,
                                            const void* v, int64_t v_stride, float q_scale, const double* log_decay,
                                            const float* log_in, const double* log_decay_sum, const float* running_max,
                                            const float* tile_max, float* state, const int32_t* cu_seqlens,
                                            const int64_t* positions, const int32_t* state_slots, const int32_t* tiles,
                                            const int32_t* tile_start, int32_t num_tiles, int32_t tile_rows, int32_t num_seqs,
                                            int32_t num_heads, int32_t head_dim, int32_t v_dim, int64_t num_tokens,
                                            float* workspace, int64_t workspace_floats, int32_t dtype, void* stream) {
  MI355_REQUIRE(o && q && k && v && state && cu_seqlens && positions && state_slots && tiles && tile_start && workspace,
                MI355_ERR_INVALID, "linear_attn_chunks: null pointer");
  const bool mem = log_decay == nullptr;
  MI355_REQUIRE(!mem || (log_in && log_decay_sum && running_max && tile_max), MI355_ERR_INVALID,
                "linear_attn_chunks: either the heads' log decay or the four gate arrays");
  MI355_REQUIRE(num_seqs >= 0 && num_seqs <= 65535 && num_tiles >= 0 && num_heads > 0 && num_heads <= 65535 && head_dim > 0 &&
                    v_dim > 0 && num_tokens >= 0,
                MI355_ERR_INVALID, "linear_attn_chunks: sizes");
  MI355_REQUIRE(q_stride >= static_cast<int64_t>(num_heads) * head_dim && k_stride >= static_cast<int64_t>(num_heads) * head_dim &&
                    v_stride >= static_cast<int64_t>(num_heads) * v_dim,
                MI355_ERR_INVALID, "linear_attn_chunks: row strides shorter than the rows");
  REQ_DTYPE(dtype);
  LaDims D{num_heads, head_dim, v_dim, static_cast<int>(la_state_floats(head_dim, v_dim, mem)), tile_rows};
  MI355_REQUIRE(tile_rows > 0 && tile_rows <= 64 && tile_rows % 16 == 0 && la_out_lds(tile_rows, head_dim, v_dim) <= kLdsBytes &&
                    la_states_lds(tile_rows, head_dim, v_dim) <= kLdsBytes,
                MI355_ERR_UNSUPPORTED, "linear_attn_chunks: tiles of %d rows of heads of %d / %d do not fit the LDS", tile_rows,
                head_dim, v_dim);
  MI355_REQUIRE(workspace_floats >= static_cast<int64_t>(num_tiles) * num_heads * (D.us + 1) && aligned16(workspace) && aligned16(state),
                MI355_ERR_INVALID, "linear_attn_chunks: workspace of %lld floats", static_cast<long long>(workspace_floats));
  if (num_seqs == 0 || num_tiles == 0 || num_tokens == 0) return MI355_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int vec = dtype != MI355_F32 && head_dim % 8 == 0 && v_dim % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 &&
                  v_stride % 8 == 0 && aligned16(q) && aligned16(k) && aligned16(v);
  const dim3 grid(num_tiles, num_heads);
  const size_t lds_states = la_states_lds(tile_rows, head_dim, v_dim), lds_out = la_out_lds(tile_rows, head_dim, v_dim);
  const dim3 sgrid((D.us / 4 + 255) / 256, num_heads, num_seqs);
#define MI355_LA(TT, MM)                                                                                                       \
  do {                                                                                                                         \
    typedef Elem<TT>::S E;                                                                                                     \
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(la_states_kernel<TT, MM>),                                         \
                              hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds_states));                       \
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(la_out_kernel<TT, MM>), hipFuncAttributeMaxDynamicSharedMemorySize, \
                              static_cast<int>(lds_out));                                                                      \
    hipLaunchKernelGGL((la_states_kernel<TT, MM>), grid, dim3(256), lds_states, s, workspace, static_cast<const E*>(k), k_stride, \
                       static_cast<const E*>(v), v_stride, log_decay, log_in, log_decay_sum, running_max, tile_max, tiles, D,  \
                       num_tokens, static_cast<int64_t>(num_tiles), vec);                                                      \
    hipLaunchKernelGGL(la_scan_kernel, sgrid, dim3(256), 0, s, workspace, state, cu_seqlens, positions, state_slots,           \
                       tile_start, D, static_cast<int64_t>(num_tiles));                                                        \
    hipLaunchKernelGGL((la_out_kernel<TT, MM>), grid, dim3(512), lds_out, s, o, workspace, static_cast<const E*>(q), q_stride, \
                       static_cast<const E*>(k), k_stride, static_cast<const E*>(v), v_stride, q_scale, log_decay, log_in,     \
                       log_decay_sum, running_max, tile_max, tiles, D, num_tokens, vec);                                       \
  } while (0)
  MI355_DISPATCH_DTYPE3(dtype, {
    if (mem) MI355_LA(TT, true); else MI355_LA(TT, false);
  });
#undef MI355_LA
  return check_launch("linear_attn_chunks");
}

static inline int64_t la_step_lds(int d, int dv) {
  const int vw = dv % 4 == 0 ? 4 : 1;
  const int nc = dv / vw, cg = nc < 256 ? nc : 256, rg = 256 / cg;
  return sizeof(float) * (2 * static_cast<int64_t>(d) + dv + static_cast<int64_t>(rg) * cg * vw);
}

template <typename TT, bool MEM>
static void launch_la_step(hipStream_t s, float* o, const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v,
                           int64_t v_stride, float q_scale, const double* log_decay, float* state, const int32_t* cu_seqlens,
                           const int64_t* positions, const int32_t* state_slots, int num_seqs, const LaDims& D,
                           const LaStepMem& M) {
  typedef typename Elem<TT>::S E;
  const dim3 grid(num_seqs, D.H);
  const size_t lds = la_step_lds(D.d, D.dv);
#define MI355_STEP(VW)                                                                                                       \
  hipLaunchKernelGGL((la_step_kernel<TT, MEM, VW>), grid, dim3(256), lds, s, o, static_cast<const E*>(q), q_stride,          \
                     static_cast<const E*>(k), k_stride, static_cast<const E*>(v), v_stride, q_scale, log_decay, state,      \
                     cu_seqlens, positions, state_slots, D, M)
  if (D.dv % 4 == 0) MI355_STEP(4);
  else MI355_STEP(1);
#undef MI355_STEP
}

static int32_t check_la_step(const char* name, const void* q, const void* k, const void* v, const float* state,
                             const int32_t* cu_seqlens, const int64_t* positions, const int32_t* state_slots, int64_t q_stride,
                             int64_t k_stride, int64_t v_stride, int num_seqs, int H, int d, int dv, int dtype) {
  MI355_REQUIRE(q && k && v && state && cu_seqlens && positions && state_slots, MI355_ERR_INVALID, "%s: null pointer", name);
  MI355_REQUIRE(num_seqs >= 0 && H > 0 && H <= 65535 && d > 0 && dv > 0 && q_stride >= static_cast<int64_t>(H) * d &&
                    k_stride >= static_cast<int64_t>(H) * d && v_stride >= static_cast<int64_t>(H) * dv && aligned16(state),
                MI355_ERR_INVALID, "%s: sizes", name);
  MI355_REQUIRE(la_step_lds(d, dv) <= 60 * 1024, MI355_ERR_UNSUPPORTED, "%s: heads of %d / %d", name, d, dv);
  REQ_DTYPE(dtype);
  return MI355_OK;
}

extern "C" int32_t mi355_decay_attn_step(float* o, const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v,
                                         int64_t v_stride, const double* log_decay, float* state, const int32_t* cu_seqlens,
                                         const int64_t* positions, const int32_t* state_slots, int32_t num_seqs,
                                         int32_t num_heads, int32_t head_dim, int32_t v_dim, int32_t dtype, void* stream) {
  MI355_REQUIRE(o && log_decay, MI355_ERR_INVALID, "decay_attn_step: null pointer");
  const int32_t rc = check_la_step("decay_attn_step", q, k, v, state, cu_seqlens, positions, state_slots, q_stride, k_stride,
                                   v_stride, num_seqs, num_heads, head_dim, v_dim, dtype);
  if (rc != MI355_OK || num_seqs == 0) return rc;
  LaDims D{num_heads, head_dim, v_dim, static_cast<int>(la_state_floats(head_dim, v_dim, false)), 0};
  MI355_DISPATCH_DTYPE3(dtype, (launch_la_step<TT, false>(static_cast<hipStream_t>(stream), o, q, q_stride, k, k_stride, v, v_stride,
                                                          1.0f, log_decay, state, cu_seqlens, positions, state_slots, num_seqs,
                                                          D, LaStepMem{})));
  return check_launch("decay_attn_step");
}

extern "C" int32_t mi355_mlstm_step(void* out, int64_t out_stride, const void* q, int64_t q_stride, const void* k, int64_t k_stride,
                                    const void* v, int64_t v_stride, float q_scale, const float* x, int64_t x_stride,
                                    const void* gate_w, const float* gate_b, int32_t width, float cap, const void* g,
                                    int64_t g_stride, const float* norm, float eps, float* state, float* m_state,
                                    const int32_t* cu_seqlens, const int64_t* positions, const int32_t* state_slots,
                                    int32_t num_seqs, int32_t num_heads, int32_t head_dim, int32_t v_dim, int32_t dtype,
                                    void* stream) {
  MI355_REQUIRE(out && x && gate_w && gate_b && g && norm && m_state, MI355_ERR_INVALID, "mlstm_step: null pointer");
  const int64_t hv = static_cast<int64_t>(num_heads) * v_dim;
  MI355_REQUIRE(out_stride >= hv && g_stride >= hv && width > 0 && x_stride >= width && cap > 0.f, MI355_ERR_INVALID,
                "mlstm_step: sizes");
  const int32_t rc = check_la_step("mlstm_step", q, k, v, state, cu_seqlens, positions, state_slots, q_stride, k_stride, v_stride,
                                   num_seqs, num_heads, head_dim, v_dim, dtype);
  if (rc != MI355_OK || num_seqs == 0) return rc;
  LaDims D{num_heads, head_dim, v_dim, static_cast<int>(la_state_floats(head_dim, v_dim, true)), 0};
  const LaStepMem M{x, x_stride, gate_w, gate_b, width, cap, m_state, g, g_stride, norm, eps, out, out_stride};
  MI355_DISPATCH_DTYPE3(dtype, (launch_la_step<TT, true>(static_cast<hipStream_t>(stream), nullptr, q, q_stride, k, k_stride, v,
                                                         v_stride, q_scale, nullptr, state, cu_seqlens, positions, state_slots,
                                                         num_seqs, D, M)));
  return check_launch("mlstm_step");
}
