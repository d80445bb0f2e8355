// H14 .. H17: a mixture of gated experts, expert by expert. fp32 accumulation throughout.
//
//   moe_sort       (row, choice) pairs grouped by expert: a pair's place, the pair at every place, and
//                  the list of tiles (expert, first place, end) the grouped products walk. One
//                  workgroup, no host round trip.
//   moe_gemm       prompts, bf16: C = A_e . B_e^T for every expert's rows in one launch of 128 x 128
//                  tiles on mfma_f32_32x32x16_bf16; the first product gathers its rows through the
//                  sorted pairs and writes silu(gate) * up (a tile holds the gate and the up columns of
//                  the same 64 hidden entries), the second writes every pair's output row.
//   moe_pairs      decode steps, bf16: a workgroup takes 16 output entries of ONE expert and all rows
//                  routed to it, so an expert's weights are read once for up to 16 rows that chose it.
//   moe_combine    out[t] = sum_k wt[t, k] * y[place of pair (t, k)], in the order of the choices
//
// A row's result does not depend on its place or on the other rows.
#include "../common.h"

namespace {

using rt::DT;

RT_DEVICE float sigm(float v) { return 1.0f / (1.0f + expf(-v)); }

constexpr int kTileM = 128, kTileN = 128, kTileK = 64;

// ---- grouping -------------------------------------------------------------------------------------

// tiles [max_tiles][3] = (expert, first place, end place); unused entries get expert -1.
// dynamic LDS: counts [E], offsets [E + 1], tile offsets [E + 1]
__global__ void __launch_bounds__(1024) moe_sort_kernel(const int* __restrict__ idx, int P, int E, int* __restrict__ place,
                                                        int* __restrict__ order, int* __restrict__ tiles, int max_tiles) {
  extern __shared__ int cnt[];
  int* off = cnt + E;
  int* toff = off + E + 1;
  for (int e = threadIdx.x; e < E; e += blockDim.x) cnt[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += blockDim.x) atomicAdd(&cnt[idx[i]], 1);
  __syncthreads();
  if (threadIdx.x < 64) {      // prefix sums: every lane of the first wave takes E / 64 neighbours
    const int per = (E + 63) / 64, lo = min(E, (int)threadIdx.x * per), hi = min(E, lo + per);
    int s = 0, t = 0;
    for (int e = lo; e < hi; ++e) {
      s += cnt[e];
      t += (cnt[e] + kTileM - 1) / kTileM;
    }
    int ps = s, pt = t;
    for (int o = 1; o < 64; o <<= 1) {
      const int a = __shfl_up(ps, o, 64), b = __shfl_up(pt, o, 64);
      if ((int)threadIdx.x >= o) {
        ps += a;
        pt += b;
      }
    }
    ps -= s;
    pt -= t;
    for (int e = lo; e < hi; ++e) {
      off[e] = ps;
      toff[e] = pt;
      ps += cnt[e];
      pt += (cnt[e] + kTileM - 1) / kTileM;
    }
    if (threadIdx.x == 63) {
      off[E] = ps;
      toff[E] = pt;
    }
  }
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += blockDim.x) {
    const int n = cnt[e];
    for (int j = 0; j * kTileM < n; ++j) {
      int* t = tiles + 3 * (toff[e] + j);
      t[0] = e;
      t[1] = off[e] + j * kTileM;
      t[2] = off[e] + n;
    }
  }
  for (int j = toff[E] + threadIdx.x; j < max_tiles; j += blockDim.x) tiles[3 * j] = -1;
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += blockDim.x) cnt[e] = off[e];
  __syncthreads();
  for (int i = threadIdx.x; i < P; i += blockDim.x) {
    const int p = atomicAdd(&cnt[idx[i]], 1);
    place[i] = p;
    order[p] = i;
  }
}

// ---- grouped products on the matrix cores ---------------------------------------------------------

typedef float f16v __attribute__((ext_vector_type(16)));

struct GroupedArgs {
  uint16_t* out;           // [pairs][N]
  const uint16_t* a;       // [rows][K]
  const uint16_t* b;       // [E][NB][K]: NB = 2 N (gate rows, then up rows) or N
  const int* tiles;
  const int* order;        // pair at every place (row = pair / top), or null: row = place
  int n_tiles, n_blocks, N, K, top;
};

constexpr int kGroupM = 4;     // neighbouring row tiles that share a weight tile while it is in the L2

// Both operands are K-contiguous rows. LDS tiles of 128 rows x 64 entries, 16-byte chunk q of row r
// at place q ^ (r & 7), so that 8 lanes reading one chunk column of 8 rows touch every bank once.
// Wave (wm, wn) owns 64 rows and two blocks of 32 columns: with GLU the gate and the up column block
// of the same hidden entries, so that silu(gate) * up needs no exchange. The next K step's chunks
// are loaded into registers while the current one is multiplied.
template <bool GLU>
__global__ void __launch_bounds__(256, 2) moe_gemm_kernel(GroupedArgs g) {
  extern __shared__ __align__(16) unsigned char smem[];      // [2][A 16 KB | B 16 KB]
  constexpr int kCols = GLU ? kTileN / 2 : kTileN;           // output columns of a tile
  // an XCD takes a contiguous range of the grouped order (workgroups go round the 8 XCDs)
  const int total = g.n_tiles * g.n_blocks;
  const int per = (total + 7) / 8;
  const int id = (int)(blockIdx.x % 8) * per + (int)(blockIdx.x / 8);
  if (id >= total || (int)(blockIdx.x / 8) >= per) return;
  const int group = id / (kGroupM * g.n_blocks), rem = id - group * kGroupM * g.n_blocks;
  const int gm = min(kGroupM, g.n_tiles - group * kGroupM);
  const int tile = group * kGroupM + rem % gm, nb = rem / gm;
  const int expert = g.tiles[3 * tile];
  if (expert < 0) return;
  const int p0 = g.tiles[3 * tile + 1], pe = min(g.tiles[3 * tile + 2], p0 + kTileM);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = lane & 31, h = lane >> 5, wm = wave >> 1, wn = wave & 1;
  const int K = g.K, N = g.N, n0 = nb * kCols;
  // staging: thread -> chunk q of rows r, r + 32, r + 64, r + 96
  const int q = tid & 7, r = tid >> 3;
  const uint16_t* ap[4];
  const uint16_t* bp[4];
  bool bok[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = r + 32 * j;
    const int place = min(p0 + row, pe - 1);                 // rows past the end repeat the last one
    const int src = g.order ? g.order[place] / g.top : place;
    ap[j] = g.a + (size_t)src * K + q * 8;
    // GLU: tile rows 0 .. 63 are gate rows n0 .., 64 .. 127 the up rows of the same entries
    const int col = GLU ? n0 + (row & 63) : n0 + row;
    bok[j] = col < N;
    const size_t brow = (size_t)expert * (GLU ? 2 : 1) * N + (GLU && row >= 64 ? N : 0) + (bok[j] ? col : 0);
    bp[j] = g.b + brow * K + q * 8;
  }
  const unsigned st = (unsigned)(r * 128 + ((q ^ (r & 7)) * 16));       // (row + 32) & 7 == row & 7
  rt::u32x4 va[4], vb[4];
  auto load = [&](int k0) {
    const bool ok = k0 + q * 8 < K;                          // K is a multiple of 8
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      va[j] = rt::u32x4{0u, 0u, 0u, 0u};
      vb[j] = rt::u32x4{0u, 0u, 0u, 0u};
      if (ok) va[j] = *reinterpret_cast<const rt::u32x4*>(ap[j] + k0);
      if (ok && bok[j]) vb[j] = *reinterpret_cast<const rt::u32x4*>(bp[j] + k0);
    }
  };
  auto store = [&](int buf) {
    unsigned char* A = smem + buf * 32768;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      *reinterpret_cast<rt::u32x4*>(A + st + j * 4096) = va[j];
      *reinterpret_cast<rt::u32x4*>(A + 16384 + st + j * 4096) = vb[j];
    }
  };
  f16v acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][j][e] = 0.f;
  const int ar0 = wm * 64 + c;
  const int br0 = GLU ? wn * 32 + c : wn * 64 + c, br1 = GLU ? 64 + wn * 32 + c : wn * 64 + 32 + c;
  const int nk = (K + kTileK - 1) / kTileK;
  load(0);
  store(0);
  if (nk > 1) load(kTileK);
  __syncthreads();
  for (int k = 0; k < nk; ++k) {
    const unsigned char* A = smem + (k & 1) * 32768;
    const unsigned char* B = A + 16384;
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const int sw = ((kk * 2 + h) ^ (c & 7)) * 16;          // every fragment row is c modulo 8
      const rt::short8 a0 = *reinterpret_cast<const rt::short8*>(A + ar0 * 128 + sw);
      const rt::short8 a1 = *reinterpret_cast<const rt::short8*>(A + (ar0 + 32) * 128 + sw);
      const rt::short8 b0 = *reinterpret_cast<const rt::short8*>(B + br0 * 128 + sw);
      const rt::short8 b1 = *reinterpret_cast<const rt::short8*>(B + br1 * 128 + sw);
      acc[0][0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a0), __builtin_bit_cast(rt::bf16x8, b0), acc[0][0], 0, 0, 0);
      acc[0][1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a0), __builtin_bit_cast(rt::bf16x8, b1), acc[0][1], 0, 0, 0);
      acc[1][0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a1), __builtin_bit_cast(rt::bf16x8, b0), acc[1][0], 0, 0, 0);
      acc[1][1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a1), __builtin_bit_cast(rt::bf16x8, b1), acc[1][1], 0, 0, 0);
    }
    if (k + 1 < nk) store((k + 1) & 1);       // its readers passed the barrier of step k - 1
    if (k + 2 < nk) load((k + 2) * kTileK);
    __syncthreads();
  }
  // register e of a block: row 8 (e >> 2) + 4 h + (e & 3), column c
#pragma unroll
  for (int i = 0; i < 2; ++i) {
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int place = p0 + wm * 64 + 32 * i + 8 * (e >> 2) + 4 * h + (e & 3);
      if (place >= pe) continue;
      uint16_t* o = g.out + (size_t)place * N;
      if (GLU) {
        const int col = n0 + wn * 32 + c;
        const float gt = acc[i][0][e];
        if (col < N) o[col] = rt::f2bf(gt * sigm(gt) * acc[i][1][e]);
      } else {
        const int col = n0 + wn * 64 + c;
        if (col < N) o[col] = rt::f2bf(acc[i][0][e]);
        if (col + 32 < N) o[col + 32] = rt::f2bf(acc[i][1][e]);
      }
    }
  }
}

// ---- decode steps: one expert's weights, every row that chose it ----------------------------------

constexpr int kPairWaves = 4, kPairBlock = 16;      // output entries of one workgroup
constexpr int kMaxPairs = 1024;

// the pairs that chose `expert`, in order (wave 0); returns their number
RT_DEVICE int list_pairs(const int* __restrict__ idx, int P, int expert, int* list, int* count) {
  if (threadIdx.x < 64) {
    int n = 0;
    for (int b = 0; b < P; b += 64) {
      const int i = b + (int)threadIdx.x;
      const bool hit = i < P && idx[i] == expert;
      const unsigned long long m = __ballot(hit);
      if (hit) list[n + __popcll(m & ((1ull << threadIdx.x) - 1ull))] = i;
      n += __popcll(m);
    }
    if (threadIdx.x == 0) *count = n;
  }
  __syncthreads();
  return *count;
}

typedef float f4v __attribute__((ext_vector_type(4)));

// grid (blocks of 16 output entries, experts). GLU: w [E][2N][K] (gate rows, up rows), input row of
// pair p = row p / top of x [T][K], out bf16 [pairs][N] = silu(gate) * up; else w [E][N][K], input
// row p of x, out fp32 [pairs][N]. The four waves take a quarter of K each: a wave streams its part of
// the 16 (32) weight rows straight into mfma_f32_16x16x32_bf16 operands — up to kUnroll steps of
// loads in flight, no LDS — against up to 16 input rows (the columns); the quarters are added
// through LDS.
template <bool GLU>
__global__ void __launch_bounds__(64 * kPairWaves) moe_pairs_kernel(void* __restrict__ out, const uint16_t* __restrict__ x,
                                                                    const uint16_t* __restrict__ w,
                                                                    const int* __restrict__ idx, int P, int top, int K,
                                                                    int N) {
  constexpr int NW = GLU ? 2 : 1;
  constexpr int kUnroll = GLU ? 4 : 8;
  __shared__ int list[kMaxPairs];
  __shared__ int count;
  __shared__ float part[kPairWaves][NW][16 * 17];      // [input row][entry], rows padded
  const int expert = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int n = list_pairs(idx, P, expert, list, &count);
  if (n == 0) return;
  const int c = lane & 15, h = lane >> 4;              // weight row / input row of this lane, its 8 entries of a step
  const int f0 = blockIdx.x * kPairBlock;
  const int frow = min(f0 + c, N - 1);
  const uint16_t* wp[NW];
#pragma unroll
  for (int j = 0; j < NW; ++j) wp[j] = w + ((size_t)expert * NW * N + (size_t)j * N + frow) * K + 8 * h;
  const int kq = ((K + 32 * kPairWaves - 1) / (32 * kPairWaves)) * 32;     // a wave's part of K: whole steps of 32
  const int kb = wave * kq, ke = min(K, kb + kq);
  for (int b = 0; b < n; b += 16) {
    const int m = min(16, n - b);
    const int pair = list[b + min(c, m - 1)];
    const uint16_t* xp = x + (size_t)(GLU ? pair / top : pair) * K + 8 * h;
    f4v acc[NW];
#pragma unroll
    for (int j = 0; j < NW; ++j) acc[j] = f4v{0.f, 0.f, 0.f, 0.f};
    for (int k = kb; k < ke; k += 32 * kUnroll) {
      rt::u32x4 wv[kUnroll][NW], xv[kUnroll];
#pragma unroll
      for (int u = 0; u < kUnroll; ++u) {
        const bool ok = k + 32 * u + 8 * h < ke;          // K is a multiple of 8
#pragma unroll
        for (int j = 0; j < NW; ++j) {
          wv[u][j] = rt::u32x4{0u, 0u, 0u, 0u};
          if (ok) wv[u][j] = *reinterpret_cast<const rt::u32x4*>(wp[j] + k + 32 * u);
        }
        xv[u] = rt::u32x4{0u, 0u, 0u, 0u};
        if (ok) xv[u] = *reinterpret_cast<const rt::u32x4*>(xp + k + 32 * u);
      }
#pragma unroll
      for (int u = 0; u < kUnroll; ++u)
#pragma unroll
        for (int j = 0; j < NW; ++j)
          acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(rt::bf16x8, wv[u][j]),
                                                           __builtin_bit_cast(rt::bf16x8, xv[u]), acc[j], 0, 0, 0);
    }
    // lane: column c (input row), rows 4 h + e (weight rows)
#pragma unroll
    for (int j = 0; j < NW; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) part[wave][j][c * 17 + 4 * h + e] = acc[j][e];
    __syncthreads();
    const int row = threadIdx.x >> 4, ent = threadIdx.x & 15;
    if (row < m && f0 + ent < N) {
      float v[NW];
#pragma unroll
      for (int j = 0; j < NW; ++j) {
        v[j] = 0.f;
#pragma unroll
        for (int q = 0; q < kPairWaves; ++q) v[j] += part[q][j][row * 17 + ent];
      }
      const size_t at = (size_t)list[b + row] * N + f0 + ent;
      if constexpr (GLU) ((uint16_t*)out)[at] = rt::f2bf(v[0] * sigm(v[0]) * v[1]);
      else ((float*)out)[at] = v[0];
    }
    __syncthreads();
  }
}

template <typename OT, typename YT>
__global__ void __launch_bounds__(256) moe_combine_kernel(OT* __restrict__ out, const YT* __restrict__ y,
                                                          const float* __restrict__ wt, const int* __restrict__ place,
                                                          int W, int top) {
  const int t = blockIdx.x;
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < W; c += blockDim.x * gridDim.y) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const int p = t * top + k;
      acc += wt[p] * DT<YT>::load(y + (size_t)(place ? place[p] : p) * W + c);
    }
    DT<OT>::store(out + (size_t)t * W + c, acc);
  }
}

}  // namespace

int moe_tile_rows() { return kTileM; }

int launch_moe_sort(const int* idx, int P, int E, int* place, int* order, int* tiles, int max_tiles, hipStream_t stream) {
  if (P <= 0) return 0;
  const size_t shm = sizeof(int) * (size_t)(3 * E + 2);
  if (shm > 48 * 1024) return -1;
  moe_sort_kernel<<<1, 1024, shm, stream>>>(idx, P, E, place, order, tiles, max_tiles);
  return 0;
}

// glu: b [E][2N][K] -> out [pairs][N] = silu(gate) * up; else b [E][N][K]. K a multiple of 8.
int launch_moe_gemm(void* out, const void* a, const void* b, const int* tiles, int n_tiles, const int* order, int N, int K,
                    int top, bool glu, hipStream_t stream) {
  if (n_tiles <= 0 || N <= 0) return 0;
  if (K % 8 || K <= 0) return -1;
  GroupedArgs g;
  g.out = (uint16_t*)out; g.a = (const uint16_t*)a; g.b = (const uint16_t*)b; g.tiles = tiles; g.order = order;
  g.n_tiles = n_tiles; g.N = N; g.K = K; g.top = top;
  const int cols = glu ? kTileN / 2 : kTileN;
  g.n_blocks = (N + cols - 1) / cols;
  const long long total = (long long)n_tiles * g.n_blocks;
  if (total > (1 << 28)) return -2;
  const int grid = (int)((total + 7) / 8 * 8);
  const int shm = 2 * 32768;
  if (glu) {
    if (hipFuncSetAttribute((const void*)moe_gemm_kernel<true>, hipFuncAttributeMaxDynamicSharedMemorySize, shm) != hipSuccess) return -3;
    moe_gemm_kernel<true><<<grid, 256, shm, stream>>>(g);
  } else {
    if (hipFuncSetAttribute((const void*)moe_gemm_kernel<false>, hipFuncAttributeMaxDynamicSharedMemorySize, shm) != hipSuccess) return -3;
    moe_gemm_kernel<false><<<grid, 256, shm, stream>>>(g);
  }
  return 0;
}

// bf16: hid [P][F] bf16 scratch, y [P][W] fp32 = every pair's output row, P = T * top <= 1024; W and F
// multiples of 8
int launch_moe_pairs(float* y, void* hid, const void* h, const void* wgu, const void* wd, const int* idx, int T, int W,
                     int F, int E, int top, hipStream_t stream) {
  if (T <= 0) return 0;
  const int P = T * top;
  if (P > kMaxPairs) return -1;
  if (W % 8 || F % 8) return -2;
  moe_pairs_kernel<true><<<dim3((F + kPairBlock - 1) / kPairBlock, E), 64 * kPairWaves, 0, stream>>>(
      hid, (const uint16_t*)h, (const uint16_t*)wgu, idx, P, top, W, F);
  moe_pairs_kernel<false><<<dim3((W + kPairBlock - 1) / kPairBlock, E), 64 * kPairWaves, 0, stream>>>(
      y, (const uint16_t*)hid, (const uint16_t*)wd, idx, P, top, F, W);
  return 0;
}

void launch_moe_combine(void* out, const void* y, const float* wt, const int* place, int T, int W, int top, bool out_bf,
                        bool y_bf, hipStream_t stream) {
  if (T <= 0) return;
  const dim3 grid(T, (W + 1023) / 1024);
#define RT_MC(OT, YT) moe_combine_kernel<OT, YT><<<grid, 256, 0, stream>>>((OT*)out, (const YT*)y, wt, place, W, top)
  if (out_bf) {
    if (y_bf) RT_MC(uint16_t, uint16_t); else RT_MC(uint16_t, float);
  } else {
    if (y_bf) RT_MC(float, uint16_t); else RT_MC(float, float);
  }
#undef RT_MC
}
