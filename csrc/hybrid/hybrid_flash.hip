// H19: the attention of H3 on the matrix cores (bf16): causal grouped-query attention over plain-row paged
// keys and values with a sliding window and kept first keys, or chunks; a soft cap; a learned sink per
// head; one gate per head; the result scaled into a column range. Head sizes are multiples of 8 up to
// 256 that need not be equal; pages are powers of two of at least 4 tokens.
//
//   K cache [num_blocks, G, BS, Dk], V cache [num_blocks, G, BS, Dv], q [T, H, Dk]
//
// A workgroup of 4 waves = one work item (sequence, first row) x one key/value head x one key range: 32
// (row, head) pairs per wave that all read the same keys, walked in tiles of 64 counted from key 0. KS = 2
// (launches too small to fill the chip with 128-pair workgroups): two waves share 32 pairs, each takes half
// of every tile's keys, and their results are merged at the end.
//
//   S^T [64 keys x 32 pairs] = K Q^T     mfma_f32_32x32x16_bf16, query fragments in registers; a K row is
//                                        read with its index bits 2 and 3 exchanged, so that a lane's score
//                                        registers are, as they stand, the operand P^T of the second product
//   O^T [Dv x 32 pairs] += V^T P^T       a lane owns one pair: mask, running maximum and sum without LDS
//
// A tile's keys go to LDS as rows, its values transposed (4 x 4 blocks turned in registers on the way);
// both are double-buffered with one barrier per tile: the next tile's global loads are in flight while
// this one is computed, the page numbers of the one after that too. Row strides of 16 bytes past a
// multiple of 64 keep the 16-byte fragment reads free of bank conflicts. Entries past Dk, Dv or the last
// key repeat valid ones: their weights or query entries are zero, or nothing reads the result.
//
// A split launch (one row per sequence) writes (o, m, l) per key range for flash_combine_kernel.
#include "../common.h"
#include "hybrid_args.h"

namespace {

using rt::short8;
using rt::float16_;
constexpr int kKT = 64;
constexpr float kNeg = -1e30f;
constexpr float kLog2e = 1.4426950408889634f, kLn2 = 0.6931471805599453f;
constexpr int kVRow = kKT * 2 + 16;       // bytes of a transposed value row

struct FlashArgs {
  uint16_t* out;
  const uint16_t *q, *kc, *vc, *gate;
  const int *block_tables, *cu_q, *start_pos, *tiles;
  float *part_o, *part_ml;
  int H, G, Dk, Dv, lgBS, max_blocks, rows, hchunks, gate_stride, out_stride, out_off, vec;
  float scale, softcap, out_scale;
  AttnMask mask;
};

// NKD, NVD: head sizes in units of 32 (padded)
template <int NKD, int NVD, int KS>
__global__ void __launch_bounds__(256) flash_kernel(FlashArgs p) {
  constexpr int NT = 256, NP = 128 / KS, NB = 2 / KS, kRow = NKD * 64 + 16, CH = NKD * 4;
  constexpr int KI = kKT * CH / NT, VI = NVD * 128 / NT;      // 16-byte key chunks, 4 x 4 value blocks per lane
  constexpr int kStage = kKT * kRow + NVD * 32 * kVRow;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 31, hi = lane >> 5;
  const int seq = p.tiles[2 * blockIdx.x], row0 = p.tiles[2 * blockIdx.x + 1];
  const int g = blockIdx.y / p.hchunks, hc = blockIdx.y - g * p.hchunks;
  const int group = p.H / p.G;
  const int h_lo = hc * NP, nh = min(group - h_lo, NP);
  const int q_lo = p.cu_q[seq];
  const int nrows = min(p.rows, p.cu_q[seq + 1] - row0);
  const int P = nrows * nh;
  const int pos0 = p.start_pos[seq] + (row0 - q_lo);
  const int kend = pos0 + nrows;
  const int S = gridDim.z;
  const TileRange tr = mask_tiles(p.mask, pos0, kend, kKT);
  const int per = (tr.n + S - 1) / S;
  const int t_lo = blockIdx.z * per, t_hi = min(tr.n, t_lo + per);
  const int BS = 1 << p.lgBS;

  // this lane's pair
  const int pw = wave % (NP / 32), kh = wave / (NP / 32);      // pairs and (KS 2) keys of this wave
  const int pair = pw * 32 + col;
  const bool mine = pair < P;
  const int pr = mine ? pair / nh : 0;
  const int h = g * group + h_lo + (mine ? pair - pr * nh : 0);
  const int row = row0 + pr, qpos = pos0 + pr, qlow = mask_low(p.mask, qpos);
  const int low_last = mask_low(p.mask, kend - 1);
  const bool busy = pw * 32 < P;

  short8 qf[NKD * 2];
  {
    const uint16_t* qr = p.q + ((size_t)row * p.H + h) * p.Dk;
#pragma unroll
    for (int c = 0; c < NKD * 2; ++c) {
      const int d = c * 16 + hi * 8;
      short8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      if (mine && d < p.Dk) z = *reinterpret_cast<const short8*>(qr + d);
      qf[c] = z;
    }
  }
  float16_ o[NVD];
#pragma unroll
  for (int d = 0; d < NVD; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[d][i] = 0.f;
  float m = kNeg, l = 0.f;

  const int* bt = p.block_tables + (size_t)seq * p.max_blocks;
  uint4 kreg[KI];
  uint2 vreg[VI][4];
  int kid[KI], vid[VI];
  auto ids = [&](int v) {          // page numbers of a tile's rows
    const int kb = tr.at(v) * kKT;
#pragma unroll
    for (int n = 0; n < KI; ++n) kid[n] = bt[min(kb + (tid + n * NT) / CH, kend - 1) >> p.lgBS];
#pragma unroll
    for (int n = 0; n < VI; ++n) {
      const int it = tid + n * NT;
      vid[n] = bt[min(kb + (((it >> 3) & 7) + ((it >> 6) & 1) * 8) * 4, kend - 1) >> p.lgBS];
    }
  };
  auto load = [&](int v) {
    const int kb = tr.at(v) * kKT;
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int it = tid + n * NT;
      const int key = min(kb + it / CH, kend - 1);
      const int d = min((it % CH) * 8, p.Dk - 8);
      kreg[n] = *reinterpret_cast<const uint4*>(p.kc + (((size_t)kid[n] * p.G + g) * BS + (key & (BS - 1))) * p.Dk + d);
    }
#pragma unroll
    for (int n = 0; n < VI; ++n) {
      const int it = tid + n * NT;
      const int d = min(((it & 7) + (it >> 7) * 8) * 4, p.Dv - 4);
      const int k0 = kb + (((it >> 3) & 7) + ((it >> 6) & 1) * 8) * 4;
      const uint16_t* base = p.vc + ((size_t)vid[n] * p.G + g) * BS * p.Dv + d;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        vreg[n][j] = *reinterpret_cast<const uint2*>(base + (size_t)(min(k0 + j, kend - 1) & (BS - 1)) * p.Dv);
    }
  };
  auto stash = [&](int buf) {
    unsigned char* ks = smem + buf * kStage;
    unsigned char* vs = ks + kKT * kRow;
#pragma unroll
    for (int n = 0; n < KI; ++n) {
      const int it = tid + n * NT;
      *reinterpret_cast<uint4*>(ks + (it / CH) * kRow + (it % CH) * 16) = kreg[n];
    }
#pragma unroll
    for (int n = 0; n < VI; ++n) {
      const int it = tid + n * NT;
      const int d = ((it & 7) + (it >> 7) * 8) * 4, kg = ((it >> 3) & 7) + ((it >> 6) & 1) * 8;
      unsigned char* at = vs + d * kVRow + kg * 8;
      const uint2 a = vreg[n][0], b = vreg[n][1], c = vreg[n][2], e = vreg[n][3];
      auto low2 = [](uint32_t x, uint32_t y) { return (x & 0xffffu) | (y << 16); };
      auto high2 = [](uint32_t x, uint32_t y) { return (x >> 16) | (y & 0xffff0000u); };
      *reinterpret_cast<uint2*>(at) = uint2{low2(a.x, b.x), low2(c.x, e.x)};
      *reinterpret_cast<uint2*>(at + kVRow) = uint2{high2(a.x, b.x), high2(c.x, e.x)};
      *reinterpret_cast<uint2*>(at + 2 * kVRow) = uint2{low2(a.y, b.y), low2(c.y, e.y)};
      *reinterpret_cast<uint2*>(at + 3 * kVRow) = uint2{high2(a.y, b.y), high2(c.y, e.y)};
    }
  };

  const int krow = (col & 0x13) | ((col & 4) << 1) | ((col & 8) >> 1);      // index bits 2 and 3 exchanged
  const float sc_in = p.softcap > 0.f ? p.scale / p.softcap * 2.f * kLog2e : p.scale * kLog2e;
  const float cap2 = p.softcap * kLog2e;

  if (t_lo < t_hi) {
    ids(t_lo);
    load(t_lo);
    if (t_lo + 1 < t_hi) ids(t_lo + 1);
    stash(0);
  }
  __syncthreads();
  for (int v = t_lo; v < t_hi; ++v) {
    const int buf = (v - t_lo) & 1;
    if (v + 1 < t_hi) {
      load(v + 1);
      if (v + 2 < t_hi) ids(v + 2);
    }
    if (busy) {
      const unsigned char* ks = smem + buf * kStage;
      const unsigned char* vs = ks + kKT * kRow;
      const int kb = tr.at(v) * kKT;
      float s[NB][16];
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        float16_ acc;
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[i] = 0.f;
#pragma unroll
        for (int c = 0; c < NKD * 2; ++c) {
          const short8 a = *reinterpret_cast<const short8*>(ks + ((kh + b) * 32 + krow) * kRow + c * 32 + hi * 16);
          acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a), __builtin_bit_cast(rt::bf16x8, qf[c]),
                                                        acc, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) s[b][i] = acc[i] * sc_in;
      }
      if (p.softcap > 0.f) {        // c tanh(x / c) = c (1 - 2 / (1 + e^(2 x / c)))
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int i = 0; i < 16; ++i)
            s[b][i] = cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(1.f + rt::fast_exp2(s[b][i]));
      }
      // a tile every row of this workgroup sees whole needs no mask
      const bool whole = kb + kKT - 1 <= pos0 && (kb >= low_last || kb + kKT <= p.mask.keep);
      float mx = kNeg;
      if (!whole) {
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int key = kb + (kh + b) * 32 + (i & 7) + hi * 8 + (i >> 3) * 16;
            if (!mask_sees(p.mask, qlow, qpos, key)) s[b][i] = 2.f * kNeg;
          }
      }
#pragma unroll
      for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int i = 0; i < 16; ++i) mx = fmaxf(mx, s[b][i]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m, mx);            // at least kNeg: an unseen key's 2 kNeg - mn stays far below zero
      const float alpha = rt::fast_exp2(m - mn);
      m = mn;
      short8 pt[2 * NB];
      float sum = 0.f;
#pragma unroll
      for (int k4 = 0; k4 < 2 * NB; ++k4) {
        float e[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          e[j] = rt::fast_exp2(s[k4 >> 1][(k4 & 1) * 8 + j] - mn);
          sum += e[j];
        }
        const uint4 w = {rt::pack2(e[0], e[1]), rt::pack2(e[2], e[3]), rt::pack2(e[4], e[5]), rt::pack2(e[6], e[7])};
        pt[k4] = __builtin_bit_cast(short8, w);
      }
      l = l * alpha + sum;
      if (__any(alpha < 1.f)) {
#pragma unroll
        for (int d = 0; d < NVD; ++d)
#pragma unroll
          for (int i = 0; i < 16; ++i) o[d][i] *= alpha;
      }
#pragma unroll
      for (int d = 0; d < NVD; ++d)
#pragma unroll
        for (int k4 = 0; k4 < 2 * NB; ++k4) {
          const short8 a = *reinterpret_cast<const short8*>(vs + (d * 32 + col) * kVRow + (2 * kh + k4) * 32 + hi * 16);
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(rt::bf16x8, a), __builtin_bit_cast(rt::bf16x8, pt[k4]),
                                                         o[d], 0, 0, 0);
        }
    }
    if (v + 1 < t_hi) stash(buf ^ 1);
    __syncthreads();
  }

  l += __shfl_xor(l, 32, 64);
  if (KS == 2) {      // (the last barrier freed the tiles) the second key half's results through LDS
    float* ex = reinterpret_cast<float*>(smem) + pw * (NVD * 16 + 2) * 64 + lane;
    if (kh == 1) {
#pragma unroll
      for (int d = 0; d < NVD; ++d)
#pragma unroll
        for (int i = 0; i < 16; ++i) ex[(d * 16 + i) * 64] = o[d][i];
      ex[NVD * 16 * 64] = m;
      ex[(NVD * 16 + 1) * 64] = l;
    }
    __syncthreads();
    if (kh == 1) return;
    const float m1 = ex[NVD * 16 * 64], M = fmaxf(m, m1);
    const float e0 = rt::fast_exp2(m - M), e1 = rt::fast_exp2(m1 - M);
    m = M;
    l = l * e0 + ex[(NVD * 16 + 1) * 64] * e1;
#pragma unroll
    for (int d = 0; d < NVD; ++d)
#pragma unroll
      for (int i = 0; i < 16; ++i) o[d][i] = o[d][i] * e0 + ex[(d * 16 + i) * 64] * e1;
  }
  if (!mine) return;
  if (S == 1) {
    float den = l, num = 1.f;
    if (p.mask.sinks) {      // relative to the larger of the two, so a sink far above the scores stays finite
      const float s2 = p.mask.sinks[h] * kLog2e, M = fmaxf(m, s2);
      num = rt::fast_exp2(m - M);
      den = l * num + rt::fast_exp2(s2 - M);
    }
    float f = den > 0.f ? num / den * p.out_scale : 0.f;
    if (p.gate) f *= 1.f / (1.f + __expf(-rt::bf2f(p.gate[(size_t)row * p.gate_stride + h])));
    uint16_t* dst = p.out + (size_t)row * p.out_stride + p.out_off + h * p.Dv;
#pragma unroll
    for (int d = 0; d < NVD; ++d)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int at = d * 32 + j * 8 + hi * 4;
        if (at >= p.Dv) continue;
        const uint2 w = {rt::pack2(o[d][4 * j] * f, o[d][4 * j + 1] * f), rt::pack2(o[d][4 * j + 2] * f, o[d][4 * j + 3] * f)};
        if (p.vec) {
          *reinterpret_cast<uint2*>(dst + at) = w;
        } else {
          dst[at] = (uint16_t)w.x; dst[at + 1] = (uint16_t)(w.x >> 16);
          dst[at + 2] = (uint16_t)w.y; dst[at + 3] = (uint16_t)(w.y >> 16);
        }
      }
  } else {
    const size_t pi = ((size_t)row * p.H + h) * S + blockIdx.z;
    float* po = p.part_o + pi * p.Dv;
#pragma unroll
    for (int d = 0; d < NVD; ++d)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int at = d * 32 + j * 8 + hi * 4;
        if (at < p.Dv) *reinterpret_cast<float4*>(po + at) = float4{o[d][4 * j], o[d][4 * j + 1], o[d][4 * j + 2], o[d][4 * j + 3]};
      }
    if (hi == 0) {
      p.part_ml[2 * pi] = m * kLn2;
      p.part_ml[2 * pi + 1] = l;
    }
  }
}

size_t flash_lds(int nkd, int nvd) { return 2 * ((size_t)kKT * (nkd * 64 + 16) + (size_t)nvd * 32 * kVRow); }

int pad_k(int D) { return D <= 64 ? 2 : D <= 96 ? 3 : D <= 128 ? 4 : 8; }
int pad_v(int D) { return D <= 64 ? 2 : D <= 128 ? 4 : 8; }

}  // namespace

void launch_gqa_combine(void* out, const float* part_o, const float* part_ml, int num_splits, int T, int H, int Dv, float sink,
                        const AttnMask& mask, const void* gate, int gate_stride, bool gate_heads, float out_scale,
                        int out_stride, int out_off, bool bf, hipStream_t stream);

int flash_key_tile() { return kKT; }

bool flash_fits(int Dk, int Dv, int BS) {
  return Dk >= 8 && Dv >= 8 && Dk <= 256 && Dv <= 256 && Dk % 8 == 0 && Dv % 8 == 0 && BS >= 4 && (BS & (BS - 1)) == 0;
}

int launch_flash_attention(void* out, const void* q, const void* kc, const void* vc, const int* block_tables, const int* cu_q,
                           const int* start_pos, const int* tiles, int n_tiles, float* part_o, float* part_ml, int T, int H,
                           int G, int Dk, int Dv, int BS, int max_blocks, int rows, int pairs, int num_splits, float scale,
                           const AttnMask& mask, const void* gate, int gate_stride, float softcap, float out_scale,
                           int out_stride, int out_off, hipStream_t stream) {
  if (n_tiles <= 0 || T <= 0) return 0;
  if (!flash_fits(Dk, Dv, BS) || H % G || (pairs != 64 && pairs != 128)) return -1;
  const int group = H / G;
  if (rows * (group < pairs ? group : pairs) > pairs) return -2;
  FlashArgs a;
  a.out = (uint16_t*)out; a.q = (const uint16_t*)q; a.kc = (const uint16_t*)kc; a.vc = (const uint16_t*)vc;
  a.gate = (const uint16_t*)gate;
  a.block_tables = block_tables; a.cu_q = cu_q; a.start_pos = start_pos; a.tiles = tiles;
  a.part_o = part_o; a.part_ml = part_ml;
  a.H = H; a.G = G; a.Dk = Dk; a.Dv = Dv; a.max_blocks = max_blocks; a.rows = rows;
  a.lgBS = 0;
  while ((1 << a.lgBS) < BS) ++a.lgBS;
  a.hchunks = (group + pairs - 1) / pairs;
  a.gate_stride = gate_stride; a.out_stride = out_stride; a.out_off = out_off;
  a.vec = out_stride % 4 == 0 && out_off % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & 7) == 0 ? 1 : 0;
  a.scale = scale; a.softcap = softcap; a.out_scale = out_scale;
  a.mask = mask;
  const dim3 grid(n_tiles, G * a.hchunks, num_splits);
  const int nk = pad_k(Dk), nv = pad_v(Dv);
  const size_t shm = flash_lds(nk, nv);
#define RT_FL(NK, NV, KSV)                                                                                             \
  do {                                                                                                                 \
    auto kern = flash_kernel<NK, NV, KSV>;                                                                             \
    if (shm > 48 * 1024 &&                                                                                             \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm) != hipSuccess)    \
      return -3;                                                                                                       \
    kern<<<grid, 256, shm, stream>>>(a);                                                                               \
  } while (0)
#define RT_FL_V(NK, KSV)                                                                                               \
  do {                                                                                                                 \
    if (nv == 2) RT_FL(NK, 2, KSV); else if (nv == 4) RT_FL(NK, 4, KSV); else RT_FL(NK, 8, KSV);                       \
  } while (0)
#define RT_FL_K(KSV)                                                                                                   \
  do {                                                                                                                 \
    if (nk == 2) RT_FL_V(2, KSV); else if (nk == 3) RT_FL_V(3, KSV); else if (nk == 4) RT_FL_V(4, KSV);                \
    else RT_FL_V(8, KSV);                                                                                              \
  } while (0)
  if (pairs == 128) RT_FL_K(1); else RT_FL_K(2);
#undef RT_FL
#undef RT_FL_V
#undef RT_FL_K
  if (num_splits > 1)
    launch_gqa_combine(out, part_o, part_ml, num_splits, T, H, Dv, 0.f, mask, gate, gate_stride, true, out_scale, out_stride,
                       out_off, true, stream);
  return 0;
}
