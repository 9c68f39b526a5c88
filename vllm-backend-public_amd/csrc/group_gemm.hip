// Grouped products on the matrix cores (16-bit storage, fp32 accumulation): for every group g
//     y = a(X_g W_g^T),   W_g [n, k],   a: the identity or relu^2
// Two kinds of groups share the kernel:
//   * a mixture's experts: group e's rows are positions offsets[e] .. offsets[e + 1] of the expert order, read
//     through perm (row perm[p] / top of x) or in place, written at their position.  The row tiles of all experts
//     are numbered by tile_start, so one launch covers whatever the loads are; no count comes to the host;
//   * heads: every group has the same rows (optionally through an index: rows of paged memory), x and y are
//     column slices x_group / y_group elements apart.
// Output addressing: y + (m / 16) * y_block + (m % 16) * y_stride + g * y_group + n, which covers plain rows
// (y_block = 16 y_stride) and pages of 16 tokens; TRANS: ... + n * 16 + m % 16 (pages with the tokens innermost).
// copy > 0: columns k .. k + copy of the x row follow the n outputs of every group (a part shared by all heads).
//
// One workgroup (4 waves) per BM x BN tile of (rows, outputs).  64-wide K steps of X and W go through registers
// into LDS: two steps on their way in registers, two images in LDS, one barrier per step.  An LDS row is 128 bytes, eight 16-byte slots; slot s of row r
// sits at s ^ ((r / 2) & 7): the 16 rows of a fragment read then cover 256 bytes without a bank twice.
#include "common.h"

namespace mi355 {

constexpr int kBK = 64;

struct GroupGemmArgs {
  uint16_t* y;
  int64_t y_block, y_stride, y_group;
  const uint16_t* x;
  int64_t x_stride, x_group, x_rows;
  const int32_t* perm;
  int top;
  const uint16_t* w;
  int64_t w_group;
  const int32_t* offsets;
  const int32_t* tile_start;
  int groups;
  int64_t rows;                        // rows of every group (heads) or of all together (experts)
  int n, k, copy, relu2;
};

// MW: waves along the rows (the other 4 / MW lie along the outputs)
template <typename T, int BM, int BN, int MW, bool TRANS>
__global__ __launch_bounds__(256, 2) void group_gemm_kernel(GroupGemmArgs a) {
  constexpr int NW = 4 / MW, TM = BM / MW / 16, TN = BN / NW / 16;      // a wave's 16 x 16 blocks
  constexpr int XP = BM * 8 / 256, WP = BN * 8 / 256;                   // 16-byte pieces per thread and step
  static_assert(BM * 8 % 256 == 0 && BN * 8 % 256 == 0, "whole pieces per thread");
  __shared__ __attribute__((aligned(16))) uint16_t lds[2][(BM + BN) * kBK];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int li = lane & 15, kk = lane >> 4;
  // workgroups go to the 8 XCDs in turn: XCD i takes the i-th contiguous part of the tiles
  const int ntn = (a.n + BN - 1) / BN;
  // (of the tiles that exist: the grid is sized for the most there can be)
  int total = gridDim.x;
  if (a.offsets != nullptr) total = min(total, MI355_LD(int32_t, a.tile_start, a.tile_start + a.groups) * ntn);
  if (static_cast<int>(blockIdx.x) >= total) return;    // (uniform over the workgroup)
  const int xcd = blockIdx.x & 7;
  const int work = xcd * (total >> 3) + min(xcd, total & 7) + (blockIdx.x >> 3);
  int mt = work / ntn;
  const int n0 = (work % ntn) * BN;
  int g;
  int64_t lo, hi;
  if (a.offsets != nullptr) {                           // the expert whose tiles hold number mt
    int l = 0, h = a.groups;                            // tile_start[l] <= mt < tile_start[h]
    while (h - l > 1) {
      const int mid = (l + h) >> 1;
      if (MI355_LD(int32_t, a.tile_start, a.tile_start + mid) <= mt) l = mid; else h = mid;
    }
    g = l;
    mt -= MI355_LD(int32_t, a.tile_start, a.tile_start + g);
    lo = MI355_LD(int32_t, a.offsets, a.offsets + g);
    hi = MI355_LD(int32_t, a.offsets, a.offsets + g + 1);
  } else {
    const int per = static_cast<int>((a.rows + BM - 1) / BM);
    g = mt / per;
    mt -= g * per;
    lo = 0;
    hi = a.rows;
  }
  const int64_t m0 = lo + static_cast<int64_t>(mt) * BM;
  if (g >= a.groups || m0 >= hi) return;
  const uint16_t* wg = a.w + g * a.w_group;
  const int r8 = tid >> 3, s8 = tid & 7;
  auto x_row = [&](int64_t p) {                          // row of x that position p reads, always a valid one
    int64_t r = p;
    if (a.perm != nullptr) r = MI355_LD(int32_t, a.perm, a.perm + p) / a.top;
    r = r < 0 ? 0 : (r >= a.x_rows ? a.x_rows - 1 : r);
    return a.x + r * a.x_stride + g * a.x_group;
  };
  const uint16_t* xp[XP];
  const uint16_t* wp[WP];
  int dx[XP], dw[WP];
#pragma unroll
  for (int j = 0; j < XP; ++j) {
    const int r = r8 + 32 * j;
    xp[j] = x_row(m0 + r < hi ? m0 + r : hi - 1);
    dx[j] = r * kBK + ((s8 ^ ((r >> 1) & 7)) << 3);
  }
#pragma unroll
  for (int j = 0; j < WP; ++j) {
    const int r = r8 + 32 * j;
    wp[j] = wg + static_cast<int64_t>(n0 + r < a.n ? n0 + r : a.n - 1) * a.k;
    dw[j] = BM * kBK + r * kBK + ((s8 ^ ((r >> 1) & 7)) << 3);
  }
  typedef unsigned int pvec __attribute__((ext_vector_type(4)));
  pvec rx[2][XP], rw[2][WP];
  // No branch around a load or a store: it would make the compiler drain the loads in flight at its join.  Columns past
  // k (the last step's, and steps past the last) read the last ones instead, and X's are cleared on the way into LDS.
  auto load = [&](int set, int t) {
    const int at = min(t * kBK + 8 * s8, a.k - 8);        // (k a multiple of 8)
#pragma unroll
    for (int j = 0; j < XP; ++j) rx[set][j] = MI355_LD(pvec, a.x, xp[j] + at);
#pragma unroll
    for (int j = 0; j < WP; ++j) rw[set][j] = MI355_LD(pvec, a.w, wp[j] + at);
  };
  auto store = [&](int set, int t) {                     // (image = set)
    const bool have = t * kBK + 8 * s8 < a.k;
#pragma unroll
    for (int j = 0; j < XP; ++j) *reinterpret_cast<pvec*>(&lds[set][dx[j]]) = have ? rx[set][j] : pvec{0, 0, 0, 0};
#pragma unroll
    for (int j = 0; j < WP; ++j) *reinterpret_cast<pvec*>(&lds[set][dw[j]]) = rw[set][j];
  };
  const int wm = (wave % MW) * (BM / MW), wn = (wave / MW) * (BN / NW);
  f32x4 acc[TM][TN];
#pragma unroll
  for (int i = 0; i < TM; ++i)
#pragma unroll
    for (int j = 0; j < TN; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int sw = (li >> 1) & 7;                          // (16-row blocks: the swizzle depends on the row in the block alone)
  const int steps = (a.k + kBK - 1) / kBK;
  load(0, 0);
  load(1, 1);
  store(0, 0);
  __syncthreads();
  // step t computes image t % 2, sends for step t + 2 and stores step t + 1 into the other image
  auto step = [&](int t, int set) {
    load(set, t + 2);
    __builtin_amdgcn_s_setprio(1);
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const int slot = ((4 * ks + kk) ^ sw) << 3;
      uint4 xf[TM], wf[TN];
#pragma unroll
      for (int i = 0; i < TM; ++i) xf[i] = *reinterpret_cast<const uint4*>(&lds[set][(wm + 16 * i + li) * kBK + slot]);
#pragma unroll
      for (int j = 0; j < TN; ++j) wf[j] = *reinterpret_cast<const uint4*>(&lds[set][BM * kBK + (wn + 16 * j + li) * kBK + slot]);
#pragma unroll
      for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j) acc[i][j] = TRANS ? T::mfma(xf[i], wf[j], acc[i][j]) : T::mfma(wf[j], xf[i], acc[i][j]);
    }
    __builtin_amdgcn_s_setprio(0);
    store(set ^ 1, t + 1);
    __syncthreads();
  };
  for (int t = 0; t < steps; t += 2) {                   // (an odd last step is followed by one of cleared X)
    step(t, 0);
    step(t + 1, 1);
  }
#pragma unroll
  for (int i = 0; i < TM; ++i) {
#pragma unroll
    for (int j = 0; j < TN; ++j) {
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        v[r] = acc[i][j][r];
        if (a.relu2) {                                   // (of the product as a 16-bit buffer would hold it)
          v[r] = fmaxf(round_f<T>(v[r]), 0.f);
          v[r] *= v[r];
        }
      }
      if (TRANS) {                                       // rows m .. m + 3 of output n
        const int64_t m = m0 + wm + 16 * i + 4 * kk;
        const int n = n0 + wn + 16 * j + li;
        if (n >= a.n || m >= hi) continue;
        uint16_t* p = a.y + (m >> 4) * a.y_block + g * a.y_group + static_cast<int64_t>(n) * 16 + (m & 15);
        if (m + 3 < hi) {
          MI355_ST(uint2, a.y, p, make_uint2(T::pack2(v[0], v[1]), T::pack2(v[2], v[3])));
        } else {
          for (int r = 0; r < 4 && m + r < hi; ++r) MI355_ST(uint16_t, a.y, p + r, T::from_f(v[r]));
        }
      } else {                                           // outputs n .. n + 3 of row m (n a multiple of 4)
        const int64_t m = m0 + wm + 16 * i + li;
        const int n = n0 + wn + 16 * j + 4 * kk;
        if (n >= a.n || m >= hi) continue;
        uint16_t* p = a.y + (m >> 4) * a.y_block + (m & 15) * a.y_stride + g * a.y_group + n;
        MI355_ST(uint2, a.y, p, make_uint2(T::pack2(v[0], v[1]), T::pack2(v[2], v[3])));
      }
    }
  }
  if (a.copy > 0 && n0 == 0) {
    const int per = a.copy >> 3;                         // 16-byte pieces per row
    for (int i = tid; i < BM * per; i += 256) {
      const int64_t m = m0 + i / per;
      if (m >= hi) break;
      const int c = (i % per) * 8;
      MI355_ST(uint4, a.y, a.y + (m >> 4) * a.y_block + (m & 15) * a.y_stride + g * a.y_group + a.n + c,
               MI355_LD(uint4, a.x, x_row(m) + a.k + c));
    }
  }
}

template <typename T>
static void launch_group_gemm(const GroupGemmArgs& a, bool trans, int64_t tiles_m, int bm, hipStream_t s) {
#define MI355_GG(BM, BN, MW, TR)                                                                                   \
  hipLaunchKernelGGL((group_gemm_kernel<T, BM, BN, MW, TR>), dim3(static_cast<unsigned>(tiles_m * ((a.n + BN - 1) / BN))), \
                     dim3(256), 0, s, a)
  if (trans) MI355_GG(128, 128, 2, true);
  else if (bm == 32) MI355_GG(32, 64, 1, false);
  else MI355_GG(128, 128, 2, false);
#undef MI355_GG
}

}  // namespace mi355

using namespace mi355;

static int32_t check_group_gemm(const char* name, const GroupGemmArgs& a, int32_t dtype) {
  MI355_REQUIRE(a.y && a.x && a.w, MI355_ERR_INVALID, "%s: null pointer", name);
  MI355_REQUIRE(dtype == MI355_BF16 || dtype == MI355_F16, MI355_ERR_UNSUPPORTED, "%s: 16-bit storage only", name);
  MI355_REQUIRE(a.groups > 0 && a.rows >= 0 && a.n > 0 && a.k > 0 && a.top > 0 && a.x_rows > 0, MI355_ERR_INVALID, "%s: sizes", name);
  MI355_REQUIRE(a.k % 8 == 0 && a.n % 4 == 0 && a.copy >= 0 && a.copy % 8 == 0 && a.x_stride % 8 == 0 && a.x_group % 8 == 0 &&
                    a.w_group % 8 == 0 && a.y_stride % 4 == 0 && a.y_block % 4 == 0 && a.y_group % 4 == 0 && aligned16(a.x) &&
                    aligned16(a.w) && aligned16(a.y),
                MI355_ERR_UNSUPPORTED, "%s: %d inputs (a multiple of 8), %d outputs (of 4), 16-byte aligned rows", name, a.k, a.n);
  MI355_REQUIRE(a.copy == 0 || (a.n % 8 == 0 && a.y_stride % 8 == 0 && a.y_block % 8 == 0 && a.y_group % 8 == 0), MI355_ERR_UNSUPPORTED,
                "%s: copied columns need outputs on 16-byte boundaries", name);
  return MI355_OK;
}

extern "C" int32_t mi355_expert_gemm(void* y, const void* x, int64_t x_rows, const void* w, const int32_t* offsets,
                                     const int32_t* tile_start, const int32_t* perm, int32_t top, int64_t num_rows,
                                     int32_t experts, int32_t out_width, int32_t in_width, int32_t relu2, int32_t dtype,
                                     void* stream) {
  MI355_REQUIRE(offsets && tile_start, MI355_ERR_INVALID, "expert_gemm: null pointer");
  GroupGemmArgs a = {static_cast<uint16_t*>(y), 16ll * out_width, out_width, 0, static_cast<const uint16_t*>(x), in_width, 0, x_rows,
                     perm, top, static_cast<const uint16_t*>(w), static_cast<int64_t>(out_width) * in_width, offsets, tile_start,
                     experts, num_rows, out_width, in_width, 0, relu2};
  const int32_t rc = check_group_gemm("expert_gemm", a, dtype);
  if (rc != MI355_OK || num_rows == 0) return rc;
  const int64_t tiles = num_rows / 128 + experts;        // no fewer than the experts' tiles together
  MI355_REQUIRE(tiles * ((out_width + 127) / 128) <= 0x7FFFFFFF, MI355_ERR_UNSUPPORTED, "expert_gemm: too many tiles");
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == MI355_BF16) launch_group_gemm<BF16>(a, false, tiles, 128, s); else launch_group_gemm<F16>(a, false, tiles, 128, s);
  return check_launch("expert_gemm");
}

extern "C" int32_t mi355_head_gemm(void* y, int64_t y_block, int64_t y_stride, int64_t y_group, const void* x, int64_t x_stride,
                                   int64_t x_group, int64_t x_rows, const int32_t* index, const void* w, int64_t num_rows,
                                   int32_t heads, int32_t out_width, int32_t in_width, int32_t copy, int32_t transposed,
                                   int32_t dtype, void* stream) {
  GroupGemmArgs a = {static_cast<uint16_t*>(y), y_block, y_stride, y_group, static_cast<const uint16_t*>(x), x_stride, x_group, x_rows,
                     index, 1, static_cast<const uint16_t*>(w), static_cast<int64_t>(out_width) * in_width, nullptr, nullptr, heads,
                     num_rows, out_width, in_width, copy, 0};
  const int32_t rc = check_group_gemm("head_gemm", a, dtype);
  if (rc != MI355_OK || num_rows == 0) return rc;
  MI355_REQUIRE(index != nullptr || x_rows >= num_rows, MI355_ERR_INVALID, "head_gemm: fewer rows than asked for");
  MI355_REQUIRE(!transposed || copy == 0, MI355_ERR_INVALID, "head_gemm: no copied columns beside transposed outputs");
  const int bm = num_rows <= 64 && !transposed ? 32 : 128;
  const int64_t tiles = ((num_rows + bm - 1) / bm) * heads;
  MI355_REQUIRE(tiles * ((out_width + 63) / 64) <= 0x7FFFFFFF, MI355_ERR_UNSUPPORTED, "head_gemm: too many tiles");
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (dtype == MI355_BF16) launch_group_gemm<BF16>(a, transposed != 0, tiles, bm, s);
  else launch_group_gemm<F16>(a, transposed != 0, tiles, bm, s);
  return check_launch("head_gemm");
}
