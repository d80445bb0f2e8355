// C5: matrix-state recurrence, fp32 throughout. Per sequence and head a D x E state S:
//
//   s = b_t^T S ;  S <- diag(w_t) S - a_t s^T + k_t v_t^T ;  o_t = S^T q_t
//
// (w: a stream per key channel, a stream per head, or one constant per head; a / b: optional removal
// streams.) This covers a constant-decay linear attention (no a / b), a matrix memory with
// exponential gates (a decay per head and token), a generalized delta rule (a = rate * unit key, b =
// unit key) and gated delta rules (w = g, a = k <- beta k, b = g k: a and k are one stream then).
//
// The token loop is a dependent chain, so its length per token is what counts. The columns of S
// are independent; a lane owns DR rows of ONE column in registers, the P = D / DR lanes of a
// column are adjacent lanes of one DPP row (P <= 16) and add their partial dot products with
// log2(P) DPP adds (quad permutes, half-row and row mirrors: no LDS crossbar). For D = 64 that is
// 4 rows per lane: about 20 FMAs and 8 DPP adds per token. One workgroup of 256 lanes =
// (sequence, head, 256 / P columns). Tokens are staged through LDS in chunks of 16: the next
// chunk's streams are loaded into registers (16-byte loads) while the current chunk is computed,
// the operands of the next token are read from LDS while the current one is computed (a whole chunk
// is unrolled over two operand sets), and a lane's share of q . S goes to LDS as it is: the shares
// of a column are added when the chunk's outputs are written, as whole lines. The state is
// kept column by column, [slot][head][E][D], so that a lane's rows are contiguous.
//
// Without removal streams (a, b) the effect of a chunk of tokens on the state is a product per key
// channel, so long spans can run in three launches over chunks: (1) every chunk alone from S = 0,
// leaving its end state and its decay product; (2) chunk by chunk, an entry of S per lane, the state
// each chunk starts from (carry = product * carry + end state, written over the end state) and the
// sequence's new state; (3) every chunk again from its true start state, writing the outputs. There is
// no division by a decay product, so decays close to zero are harmless. With removal streams the effect
// is a D x D matrix per chunk: launch (1) also runs D columns that start as the identity and get no
// values, which end as that matrix, and launch (2) multiplies by it.
#include "../common.h"

namespace {

constexpr int kScanThreads = 256;
constexpr int kTT = 16;           // tokens per staged chunk

template <int CTRL>
RT_DEVICE float dpp_add(float v) {
  const int x = __builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, true);
  return v + __int_as_float(x);
}
// sum over the P adjacent lanes of a column (P a power of two <= 16, groups aligned to P)
RT_DEVICE float group_sum(float v, int P) {
  if (P >= 2) v = dpp_add<0xB1>(v);      // quad_perm [1, 0, 3, 2]
  if (P >= 4) v = dpp_add<0x4E>(v);      // quad_perm [2, 3, 0, 1]
  if (P >= 8) v = dpp_add<0x141>(v);     // row_half_mirror (quads are uniform by now)
  if (P >= 16) v = dpp_add<0x140>(v);    // row_mirror (half rows are uniform by now)
  return v;
}

// four consecutive entries r .. r + 3 of a row of D floats (zeros from D on)
RT_DEVICE float4 load4(const float* __restrict__ row, int r, int D, bool vec) {
  if (vec && r + 3 < D) return *reinterpret_cast<const float4*>(row + r);
  float4 o;
  o.x = r < D ? row[r] : 0.f;
  o.y = r + 1 < D ? row[r + 1] : 0.f;
  o.z = r + 2 < D ? row[r + 2] : 0.f;
  o.w = r + 3 < D ? row[r + 3] : 0.f;
  return o;
}

// UNROLL: whole chunks run unrolled (prompts); without it the code is a fraction of the size, which is
// what a launch over single rows (a decode step, cold instruction cache) is timed by
// MODE 0: whole spans, state in and out of the slots; 1 / 2: launch (1) / (3) of the chunked form
// W: 0 a constant per head, 1 a decay per head and key channel, 2 a decay per head; AB: 0 no removal,
// 1 streams a and b, 2 a is the stream k. EC: columns kept per chunk and head in ws_e
template <int DR, int W, int AB, bool UNROLL, int MODE>
__global__ void __launch_bounds__(kScanThreads) state_scan_kernel(
    float* __restrict__ out, const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ v,
    const float* __restrict__ w, const float* __restrict__ a, const float* __restrict__ b, int sq, int sk, int sv, int sw,
    int sa, int sb, const float* __restrict__ decay, float* __restrict__ state, const int* __restrict__ cu_q,
    const int* __restrict__ start_pos, const int* __restrict__ slots, int A, int D, int E, int P, int lgP, int vec,
    const int* __restrict__ chunks, int chunk_rows, float* __restrict__ ws_e, float* __restrict__ ws_p, int EC) {
  extern __shared__ float4 lds4[];
  constexpr bool HAS_W = W == 1, HAS_AB = AB != 0, HAS_A = AB == 1;
  constexpr bool WIDE = MODE == 1 && HAS_AB;    // the identity's columns run too
  constexpr bool PROD = MODE == 1 && !HAS_AB;   // the chunk's decay product is kept
  constexpr bool OUT = MODE != 1;               // q is read and outputs are written
  constexpr int NQ = OUT ? 1 : 0;
  constexpr int NS = NQ + 1 + (HAS_W ? 1 : 0) + (HAS_A ? 1 : 0) + (HAS_AB ? 1 : 0);
  constexpr int NL = (kTT * DR + 63) / 64;      // 16-byte loads per lane, stream and chunk (P <= 16)
  constexpr int R4 = DR / 4;
  const int seq = MODE == 0 ? (int)blockIdx.x : chunks[2 * blockIdx.x], head = blockIdx.y;
  const int CB = kScanThreads >> lgP;           // columns of this workgroup
  const int Dp4 = (P * DR) >> 2;                // padded rows / 4 (a power of two)
  const int lgDp4 = lgP + (DR == 4 ? 0 : DR == 8 ? 1 : 2);
  const int cl = threadIdx.x >> lgP, part = threadIdx.x & (P - 1);
  const int col = blockIdx.z * CB + cl;
  const int r0 = MODE == 0 ? cu_q[seq] : chunks[2 * blockIdx.x + 1];
  const int n = MODE == 0 ? cu_q[seq + 1] - r0 : min(chunk_rows, cu_q[seq + 1] - r0);
  if (n <= 0) return;
  float4* str = lds4;                                             // [kTT][NS][Dp4]
  float* vs = reinterpret_cast<float*>(str + kTT * NS * Dp4);     // [kTT][CB]
  float* os = vs + kTT * CB;                                      // [kTT][256]: every lane's share of q . S
  float* whs = os + kTT * kScanThreads;                           // [kTT]: W 2's decays
  const int row_lo = part * DR;
  const bool live = col < (WIDE ? EC : E);
  float S[DR];
  float* sp = MODE == 0 ? state + (size_t)slots[seq] * A * E * D + ((size_t)head * E + (live ? col : 0)) * D + row_lo
                        : ws_e + (((size_t)blockIdx.x * A + head) * EC + (live ? col : 0)) * D + row_lo;
  const bool cont = MODE == 0 ? start_pos[seq] > 0 : MODE == 2;
  const bool svec = (D & 3) == 0;
#pragma unroll
  for (int i4 = 0; i4 < R4; ++i4) {
    float4 t = {0.f, 0.f, 0.f, 0.f};
    if (cont && live) t = load4(sp, i4 * 4, D - row_lo, svec);
    S[i4 * 4] = t.x; S[i4 * 4 + 1] = t.y; S[i4 * 4 + 2] = t.z; S[i4 * 4 + 3] = t.w;
  }
  if (WIDE) {
#pragma unroll
    for (int i = 0; i < DR; ++i) S[i] = col - E == row_lo + i ? 1.f : 0.f;
  }
  float prod[PROD ? DR : 1];                    // product of the chunk's decays, per row
#pragma unroll
  for (int i = 0; i < (PROD ? DR : 1); ++i) prod[i] = 1.f;
  const float dconst = W == 0 ? decay[head] : 1.f;
  const float* src[NS];
  int strides[NS];
  {
    int j = 0;
    if (OUT) { src[j] = q; strides[j++] = sq; }
    src[j] = k; strides[j++] = sk;
    if (HAS_W) { src[j] = w; strides[j++] = sw; }
    if (HAS_A) { src[j] = a; strides[j++] = sa; }
    if (HAS_AB) { src[j] = b; strides[j++] = sb; }
  }
  float4 pre[NS][NL];
  float prev[kTT];        // this lane's share of the chunk's value columns: kTT / P entries
  float prew = 1.f;
  const int nv = kTT >> lgP;      // 0 when P > kTT cannot happen (P <= 16 = kTT)
  auto fetch = [&](int c0) {
    const int nt = min(kTT, n - c0);
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const float* base = src[j] + (size_t)(r0 + c0) * strides[j] + head * D;
#pragma unroll
      for (int l = 0; l < NL; ++l) {
        const int i = threadIdx.x + l * kScanThreads;
        const int tok = i >> lgDp4, r4 = i & (Dp4 - 1);
        float4 t = {0.f, 0.f, 0.f, 0.f};
        if (tok < nt) t = load4(base + (size_t)tok * strides[j], r4 * 4, D, vec != 0);
        pre[j][l] = t;
      }
    }
#pragma unroll
    for (int l = 0; l < kTT; ++l) {
      if (l < nv) {
        const int i = threadIdx.x + l * kScanThreads;
        const int tok = i / CB, c = i - tok * CB;
        const int gc = blockIdx.z * CB + c;
        prev[l] = (tok < nt && gc < E) ? v[(size_t)(r0 + c0 + tok) * sv + head * E + gc] : 0.f;
      }
    }
    if (W == 2 && (int)threadIdx.x < nt) prew = w[(size_t)(r0 + c0 + threadIdx.x) * sw + head];
  };
  fetch(0);
  for (int c0 = 0; c0 < n; c0 += kTT) {
    const int nt = min(kTT, n - c0);
    __syncthreads();      // the previous chunk's readers are done
#pragma unroll
    for (int j = 0; j < NS; ++j) {
#pragma unroll
      for (int l = 0; l < NL; ++l) {
        const int i = threadIdx.x + l * kScanThreads;
        const int tok = i >> lgDp4, r4 = i & (Dp4 - 1);
        if (tok < kTT) str[(tok * NS + j) * Dp4 + r4] = pre[j][l];
      }
    }
#pragma unroll
    for (int l = 0; l < kTT; ++l)
      if (l < nv) vs[threadIdx.x + l * kScanThreads] = prev[l];
    if (W == 2 && threadIdx.x < kTT) whs[threadIdx.x] = prew;
    __syncthreads();
    if (c0 + kTT < n) fetch(c0 + kTT);      // in flight while this chunk is computed
    // One token: s = b . S (summed over the column's lanes, the only cross-lane step on the chain),
    // the update, and this lane's share of q . S, which goes to LDS as it is: the shares of a
    // column are added when the chunk's outputs are written, not inside the token loop.
    auto step = [&](int tok, const float4* tq, const float4* tk, const float4* tw, const float4* ta, const float4* tb,
                    float vv, float wh) {
      float sv_ = 0.f;
      if (HAS_AB) {
#pragma unroll
        for (int i4 = 0; i4 < R4; ++i4) {
          const float4 bb = tb[i4];
          sv_ += bb.x * S[i4 * 4] + bb.y * S[i4 * 4 + 1] + bb.z * S[i4 * 4 + 2] + bb.w * S[i4 * 4 + 3];
        }
        sv_ = group_sum(sv_, P);
      }
      if (AB == 2) vv -= sv_;
      float acc = 0.f;
#pragma unroll
      for (int i4 = 0; i4 < R4; ++i4) {
        const float4 kk = tk[i4];
        float u0 = kk.x * vv, u1 = kk.y * vv, u2 = kk.z * vv, u3 = kk.w * vv;
        if (HAS_A) {
          const float4 aa = ta[i4];
          u0 -= aa.x * sv_; u1 -= aa.y * sv_; u2 -= aa.z * sv_; u3 -= aa.w * sv_;
        }
        const float dh = W == 2 ? wh : dconst;
        float d0 = dh, d1 = dh, d2 = dh, d3 = dh;
        if (HAS_W) {
          const float4 ww = tw[i4];
          d0 = ww.x; d1 = ww.y; d2 = ww.z; d3 = ww.w;
        }
        S[i4 * 4] = S[i4 * 4] * d0 + u0;
        S[i4 * 4 + 1] = S[i4 * 4 + 1] * d1 + u1;
        S[i4 * 4 + 2] = S[i4 * 4 + 2] * d2 + u2;
        S[i4 * 4 + 3] = S[i4 * 4 + 3] * d3 + u3;
        if (OUT) {
          const float4 qq = tq[i4];
          acc += qq.x * S[i4 * 4] + qq.y * S[i4 * 4 + 1] + qq.z * S[i4 * 4 + 2] + qq.w * S[i4 * 4 + 3];
        }
        if constexpr (PROD) {
          prod[i4 * 4] *= d0; prod[i4 * 4 + 1] *= d1; prod[i4 * 4 + 2] *= d2; prod[i4 * 4 + 3] *= d3;
        }
      }
      if (OUT) os[tok * kScanThreads + threadIdx.x] = acc;
    };
    auto read_tok = [&](int tok, float4* tq, float4* tk, float4* tw, float4* ta, float4* tb, float& tv, float& th) {
      const float4* qs = str + (tok * NS) * Dp4 + part * R4;
      const float4* ks = qs + NQ * Dp4;
      const float4* ws = ks + Dp4;                              // HAS_W
      const float4* as = ks + (HAS_W ? 2 : 1) * Dp4;            // HAS_A
      const float4* bs = as + (HAS_A ? Dp4 : 0);                // HAS_AB
#pragma unroll
      for (int i4 = 0; i4 < R4; ++i4) {
        if (OUT) tq[i4] = qs[i4];
        tk[i4] = ks[i4];
        if (HAS_W) tw[i4] = ws[i4];
        if (HAS_A) ta[i4] = as[i4];
        if (HAS_AB) tb[i4] = bs[i4];
      }
      tv = vs[tok * CB + cl];
      if (W == 2) th = whs[tok];
    };
    if (UNROLL && nt == kTT) {
      // a whole chunk: unrolled, two operand sets in turn, so the operands of token tok + 1 are
      // read from LDS while token tok is computed and nothing is copied
      float4 oq[2][R4], ok[2][R4], ow[2][R4], oa[2][R4], ob[2][R4];
      float ov[2], oh[2] = {1.f, 1.f};
      read_tok(0, oq[0], ok[0], ow[0], oa[0], ob[0], ov[0], oh[0]);
#pragma unroll
      for (int tok = 0; tok < kTT; ++tok) {
        const int c = tok & 1, nx = c ^ 1;
        if (tok + 1 < kTT) read_tok(tok + 1, oq[nx], ok[nx], ow[nx], oa[nx], ob[nx], ov[nx], oh[nx]);
        step(tok, oq[c], ok[c], ow[c], oa[c], ob[c], ov[c], oh[c]);
      }
    } else {
      float4 tq[R4], tk[R4], tw[R4], ta[R4], tb[R4];
      float tv, th = 1.f;
      for (int tok = 0; tok < nt; ++tok) {
        read_tok(tok, tq, tk, tw, ta, tb, tv, th);
        step(tok, tq, tk, tw, ta, tb, tv, th);
      }
    }
    if (!OUT) continue;
    __syncthreads();
    for (int i = threadIdx.x; i < nt * CB; i += kScanThreads) {
      const int tok = i / CB, c = i - tok * CB;
      const int gc = blockIdx.z * CB + c;
      const float* sh = os + tok * kScanThreads + c * P;      // the column's P shares
      float o = 0.f;
      // (starting at different shares keeps the lanes of a wave on different LDS banks)
      for (int j = 0; j < P; ++j) o += sh[(j + c + tok) & (P - 1)];
      if (gc < E) out[(size_t)(r0 + c0 + tok) * A * E + head * E + gc] = o;
    }
  }
  if (MODE == 2) return;      // the sequence's new state came out of the carry
  if (PROD && blockIdx.z == 0 && cl == 0) {
    float* pp = ws_p + ((size_t)blockIdx.x * A + head) * D + row_lo;
#pragma unroll
    for (int i = 0; i < DR; ++i)
      if (row_lo + i < D) pp[i] = prod[PROD ? i : 0];
  }
  if (live) {
    if (svec && row_lo + DR <= D) {
#pragma unroll
      for (int i4 = 0; i4 < R4; ++i4) {
        float4 t = {S[i4 * 4], S[i4 * 4 + 1], S[i4 * 4 + 2], S[i4 * 4 + 3]};
        *reinterpret_cast<float4*>(sp + i4 * 4) = t;
      }
    } else {
#pragma unroll
      for (int i = 0; i < DR; ++i)
        if (row_lo + i < D) sp[i] = S[i];
    }
  }
}

// launch (2): grid (sequences, heads, blocks of 256 entries of S); a batch of chunks is loaded ahead of
// the dependent chain
constexpr int kCarryBatch = 8;
__global__ void __launch_bounds__(256) state_carry_kernel(float* __restrict__ ws_e, const float* __restrict__ ws_p,
                                                          float* __restrict__ state, const int* __restrict__ seq_chunk0,
                                                          const int* __restrict__ start_pos, const int* __restrict__ slots,
                                                          int A, int D, int E) {
  const int s = blockIdx.x, h = blockIdx.y;
  const int e = blockIdx.z * blockDim.x + threadIdx.x;      // entry col * D + row
  const int DE = D * E;
  const int k0 = seq_chunk0[s], k1 = seq_chunk0[s + 1];
  if (e >= DE || k1 <= k0) return;
  const int row = e % D;
  float* st = state + ((size_t)slots[s] * A + h) * DE + e;
  float S = start_pos[s] > 0 ? *st : 0.f;
  for (int c0 = k0; c0 < k1; c0 += kCarryBatch) {
    float end[kCarryBatch], pr[kCarryBatch];
#pragma unroll
    for (int j = 0; j < kCarryBatch; ++j) {
      const size_t at = (size_t)min(c0 + j, k1 - 1) * A + h;
      end[j] = ws_e[at * DE + e];
      pr[j] = ws_p[at * D + row];
    }
#pragma unroll
    for (int j = 0; j < kCarryBatch; ++j)
      if (c0 + j < k1) {
        ws_e[((size_t)(c0 + j) * A + h) * DE + e] = S;
        S = pr[j] * S + end[j];
      }
  }
  *st = S;
}

// launch (2) with removal: per (sequence, head, 4 * 256 / D columns) the chain S <- M_c S + B_c over the
// chunks, ws_e[chunk][head][E columns of B, then D columns of M][D]; the state a chunk starts from is
// written over its B. Lane = (row i, a group of 4 columns): it reads row i of M (coalesced over i), the
// columns of S sit in LDS. The next chunk's row of M is loaded into registers while this one is used.
template <int D>
__global__ void __launch_bounds__(256, 1) state_carry_matrix_kernel(float* __restrict__ ws_e, float* __restrict__ state,
                                                                    const int* __restrict__ seq_chunk0,
                                                                    const int* __restrict__ start_pos,
                                                                    const int* __restrict__ slots, int A, int E) {
  constexpr int groups = 256 / D;
  __shared__ float4 cols[2][D][groups];
  const int s = blockIdx.x, h = blockIdx.y;
  const int k0 = seq_chunk0[s], k1 = seq_chunk0[s + 1];
  if (k1 <= k0) return;
  const int i = threadIdx.x % D, g = threadIdx.x / D;
  const int col = (blockIdx.z * groups + g) * 4;
  const size_t step = (size_t)A * (E + D) * D;      // floats from a chunk to the next
  float* base = ws_e + (size_t)k0 * step + (size_t)h * (E + D) * D;
  float* st = state + ((size_t)slots[s] * A + h) * E * D;
  const bool cont = start_pos[s] > 0;
  int off[4];                                       // this lane's entries of B and of the state
  bool live[4];
  float S[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    live[c] = col + c < E;
    off[c] = (live[c] ? col + c : E - 1) * D + i;
    S[c] = cont && live[c] ? st[off[c]] : 0.f;
  }
  const int moff = E * D + i;
  float m[D], b[4], mn[D], bn[4];
  auto load = [&](const float* at, float (&mm)[D], float (&bb)[4]) {
#pragma unroll
    for (int c = 0; c < 4; ++c) bb[c] = at[off[c]];
    const float* row = at + moff;
#pragma unroll
    for (int j = 0; j < D; ++j) mm[j] = row[j * D];
  };
  load(base, m, b);
  for (int k = k0; k < k1; ++k, base += step) {
    float4 (*cur)[groups] = cols[(k - k0) & 1];
    cur[i][g] = float4{S[0], S[1], S[2], S[3]};
    __syncthreads();      // (the other buffer's readers are past the barrier of the step before)
    load(k + 1 < k1 ? base + step : base, mn, bn);
    float acc[4] = {b[0], b[1], b[2], b[3]};
#pragma unroll
    for (int j = 0; j < D; ++j) {
      const float4 sj = cur[j][g];
      acc[0] += m[j] * sj.x; acc[1] += m[j] * sj.y; acc[2] += m[j] * sj.z; acc[3] += m[j] * sj.w;
    }
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      if (live[c]) base[off[c]] = S[c];
      S[c] = acc[c];
      b[c] = bn[c];
    }
#pragma unroll
    for (int j = 0; j < D; ++j) m[j] = mn[j];
  }
#pragma unroll
  for (int c = 0; c < 4; ++c)
    if (live[c]) st[off[c]] = S[c];
}

// the same for any D <= 256, read as it goes
__global__ void __launch_bounds__(256) state_carry_matrix_any_kernel(float* __restrict__ ws_e, float* __restrict__ state,
                                                                     const int* __restrict__ seq_chunk0,
                                                                     const int* __restrict__ start_pos,
                                                                     const int* __restrict__ slots, int A, int D, int E) {
  extern __shared__ float4 cols[];      // [2][D]
  const int s = blockIdx.x, h = blockIdx.y, i = threadIdx.x, col = blockIdx.z * 4;
  const int k0 = seq_chunk0[s], k1 = seq_chunk0[s + 1];
  if (k1 <= k0) return;
  const int EC = E + D;
  const bool row = i < D;
  float* st = state + ((size_t)slots[s] * A + h) * E * D;
  const bool cont = start_pos[s] > 0;
  float S[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) S[c] = cont && row && col + c < E ? st[(size_t)(col + c) * D + i] : 0.f;
  for (int k = k0; k < k1; ++k) {
    float4* cur = cols + ((k - k0) & 1) * D;
    if (row) cur[i] = float4{S[0], S[1], S[2], S[3]};
    __syncthreads();
    if (row) {
      float* base = ws_e + ((size_t)k * A + h) * EC * D;
      float acc[4];
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[c] = col + c < E ? base[(size_t)(col + c) * D + i] : 0.f;
#pragma unroll 16
      for (int j = 0; j < D; ++j) {
        const float4 sj = cur[j];
        const float mj = base[(size_t)(E + j) * D + i];
        acc[0] += mj * sj.x; acc[1] += mj * sj.y; acc[2] += mj * sj.z; acc[3] += mj * sj.w;
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        if (col + c < E) base[(size_t)(col + c) * D + i] = S[c];
        S[c] = acc[c];
      }
    }
  }
#pragma unroll
  for (int c = 0; c < 4; ++c)
    if (row && col + c < E) st[(size_t)(col + c) * D + i] = S[c];
}

}  // namespace

// rows of a column one lane keeps, and lanes per column (a power of two <= 16), for D state rows
static void scan_shape(int D, int& DR, int& P, int& lgP) {
  DR = D <= 64 ? 4 : D <= 128 ? 8 : 16;
  P = 1;
  lgP = 0;
  while (P * DR < D) {
    P <<= 1;
    ++lgP;
  }
}

int launch_state_scan(float* out, const float* q, const float* k, const float* v, const float* w, const float* a,
                      const float* b, int sq, int sk, int sv, int sw, int sa, int sb, const float* decay, float* state,
                      const int* cu_q, const int* start_pos, const int* slots, int S, int T, int A, int D, int E,
                      const int* chunks, int n_chunks, int chunk_rows, const int* seq_chunk0, float* ws,
                      bool head_decay, hipStream_t stream) {
  if (S <= 0) return 0;
  if (chunks != nullptr && n_chunks <= 0) return 0;
  const bool unroll = T > 2 * S;      // rows per span on average: single rows take the small kernel
  int DR, P, lgP;
  scan_shape(D, DR, P, lgP);
  if (P > 16 || D < 1 || E < 1) return -1;
  const bool has_w = w != nullptr && !head_decay, has_ab = a != nullptr && b != nullptr;
  const bool a_is_k = has_ab && a == k && sa == sk;
  if (w == nullptr && decay == nullptr) return -2;
  if (!has_w && has_ab) return -4;
  const int NS = 2 + (has_w ? 1 : 0) + (has_ab ? (a_is_k ? 1 : 2) : 0);
  const int CB = kScanThreads / P, Dp = P * DR;
  // 16-byte loads of the streams: every row start and the head offset on a 16-byte boundary
  auto al = [&](const float* p, int st) { return p == nullptr || ((reinterpret_cast<uintptr_t>(p) & 15) == 0 && (st & 3) == 0); };
  const int vec = (D & 3) == 0 && al(q, sq) && al(k, sk) && (head_decay || al(w, sw)) && al(a, sa) && al(b, sb) ? 1 : 0;
  const size_t shm = sizeof(float) * (size_t)kTT * ((size_t)NS * Dp + CB + kScanThreads + 1);
  const int EC = has_ab ? E + D : E;      // columns per chunk and head in the scratch
  const dim3 grid_e(chunks != nullptr ? n_chunks : S, A, (E + CB - 1) / CB), grid_w(n_chunks, A, (EC + CB - 1) / CB);
  float* ws_e = ws;
  float* ws_p = ws != nullptr ? ws + (size_t)n_chunks * A * E * D : nullptr;
#define RT_SCAN(DRV, HW, HAB)                                                                                          \
  do {                                                                                                                 \
    if (unroll) RT_SCAN_U(DRV, HW, HAB, true, 0); else RT_SCAN_U(DRV, HW, HAB, false, 0);                              \
  } while (0)
#define RT_SCAN_U(DRV, HW, HAB, UN, MODE)                                                                              \
  do {                                                                                                                 \
    auto kern = state_scan_kernel<DRV, HW, HAB, UN, MODE>;                                                             \
    if (shm > 48 * 1024 &&                                                                                             \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm) != hipSuccess)    \
      return -3;                                                                                                       \
    kern<<<MODE == 1 ? grid_w : grid_e, kScanThreads, shm, stream>>>(out, q, k, v, w, a, b, sq, sk, sv, sw, sa, sb,    \
                                                                     decay, state, cu_q, start_pos, slots, A, D, E, P, \
                                                                     lgP, vec, chunks, chunk_rows, ws_e, ws_p, EC);    \
  } while (0)
#define RT_SCAN_DR(HW, HAB)                                                                                            \
  do {                                                                                                                 \
    if (DR == 4) RT_SCAN(4, HW, HAB); else if (DR == 8) RT_SCAN(8, HW, HAB); else RT_SCAN(16, HW, HAB);                \
  } while (0)
#define RT_CHUNK(HW, HAB, MODE)                                                                                        \
  do {                                                                                                                 \
    if (DR == 4) RT_SCAN_U(4, HW, HAB, true, MODE); else if (DR == 8) RT_SCAN_U(8, HW, HAB, true, MODE);               \
    else RT_SCAN_U(16, HW, HAB, true, MODE);                                                                           \
  } while (0)
#define RT_ANY(LAUNCH, ...)                                                                                            \
  do {                                                                                                                 \
    if (has_ab && a_is_k) LAUNCH(1, 2, ##__VA_ARGS__); else if (has_ab) LAUNCH(1, 1, ##__VA_ARGS__);                   \
    else if (has_w) LAUNCH(1, 0, ##__VA_ARGS__); else if (head_decay) LAUNCH(2, 0, ##__VA_ARGS__);                     \
    else LAUNCH(0, 0, ##__VA_ARGS__);                                                                                  \
  } while (0)
  if (chunks != nullptr) {
    RT_ANY(RT_CHUNK, 1);
    if (has_ab) {
      auto grid = [&](int d) { return dim3(S, A, (E + 1024 / d - 1) / (1024 / d)); };
      if (D == 64) state_carry_matrix_kernel<64><<<grid(64), 256, 0, stream>>>(ws_e, state, seq_chunk0, start_pos, slots, A, E);
      else if (D == 32) state_carry_matrix_kernel<32><<<grid(32), 256, 0, stream>>>(ws_e, state, seq_chunk0, start_pos, slots, A, E);
      else state_carry_matrix_any_kernel<<<dim3(S, A, (E + 3) / 4), 256, sizeof(float4) * 2 * (size_t)D, stream>>>(
          ws_e, state, seq_chunk0, start_pos, slots, A, D, E);
    } else {
      state_carry_kernel<<<dim3(S, A, (D * E + 255) / 256), 256, 0, stream>>>(ws_e, ws_p, state, seq_chunk0, start_pos,
                                                                              slots, A, D, E);
    }
    RT_ANY(RT_CHUNK, 2);
    return 0;
  }
  RT_ANY(RT_SCAN_DR);
#undef RT_ANY
#undef RT_SCAN_DR
#undef RT_CHUNK
#undef RT_SCAN
#undef RT_SCAN_U
  return 0;
}
