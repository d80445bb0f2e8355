// C1 - C4, C6 - C8: the row-wise kernels around input convolutions, whole-projection norms and
// matrix-state recurrences. All math fp32; activations are bf16 (uint16_t storage) or fp32 as
// templated; the residual stream, the convolution states and everything that enters a recurrence
// are fp32. One workgroup per row (256 lanes), rows are re-read from L1 / L2, so any width runs.
//
//   canon_add        xs = x + (y + y2) / rms(y + y2) * nw ; h_t = xs_t + sum_k cw[:, taps-1-k] xs_(t-k)
//                    rows ahead of a span come from the sequence's state slot, zeros ahead of position 0
//   conv_state       shift a sequence's convolution state by its rows of this batch
//   qkv_prep_wide    biases, RMS norm over the whole query / key row with a weight per channel,
//                    rotation in halves (cos / sin times a magnitude), values turned by their
//                    position or taken from the biased keys; keys / values -> the paged cache
//   turn_back        attention output turned in halves by minus the position, scaled
//   silu_cols        fp32 silu of a column range
//   removal_prep     r, k, v, decay, removal rate * unit key, unit key of a generalized delta rule
//   delta_prep       short convolutions + silu, unit q / k, step size and decay of a gated delta rule
//   gla_prep         scaled q, k, v and the decay sigmoid(low-rank path + bias)^(1 / tau) of a gated
//                    linear attention
//   channel_delta    as delta_prep, with one decay per head and key channel from a low-rank path
//   memory_gates     log input / forget gates of a matrix memory and their running maximum over a span
//   memory_prep      scaled q, weighted k, decay, v (and the column of ones that carries n)
//   head_norm_gate   per-head or whole-row RMS norm, weight, sigmoid / silu gate, scale; optionally a
//                    matrix memory's read-out, divided by max(|n . q|, exp(-m)) + 1e-6 first
//   relu2            relu(a)^2
#include "../common.h"

namespace {

using rt::DT;
constexpr int kMaxTaps = 16;
constexpr int kThreads = 256;

RT_DEVICE float sigm(float x) { return 1.0f / (1.0f + __expf(-x)); }
RT_DEVICE float silu(float x) { return x * sigm(x); }

// tap k of row t reads k tokens back: kind 1 = row t - k of this batch, 2 = the state, 0 = zeros
struct Tap {
  int kind;
  size_t at;      // kind 1: row index; kind 2: state row
};
RT_DEVICE Tap tap_of(int k, int t, int local, int64_t pos, int taps) {
  Tap r;
  r.kind = 0;
  r.at = 0;
  if (local >= k) {
    r.kind = 1;
    r.at = (size_t)(t - k);
  } else if (pos >= k) {
    r.kind = 2;
    r.at = (size_t)(taps - 1 - k + local);
  }
  return r;
}

// state layout: state[slot][sub][i][W], i < keep (= max(taps - 1, 1) rows), oldest first: row i of a
// sequence whose span starts at position p0 holds the input of position p0 - (taps - 1) + i.
// TAPS: the taps as a compile-time number (0: no convolution, only the add), or kMaxTaps for any
// number up to that (`taps` at run time)
template <typename OT, typename YT, int TAPS>
__global__ void __launch_bounds__(1024) canon_add_kernel(
    OT* __restrict__ h, float* __restrict__ xs, const float* __restrict__ x, const YT* __restrict__ y,
    const YT* __restrict__ y2, const float* __restrict__ nw, float eps, const float* __restrict__ cw,
    float* __restrict__ state, int sub, int nsub, const int* __restrict__ row_seq, const int64_t* __restrict__ positions,
    const int* __restrict__ start_pos, const int* __restrict__ slots, int W, int taps, int keep, int shift_state) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  // (loops over the taps are unrolled with a guard, so that per-tap values stay in registers)
  constexpr int NT = TAPS == 0 ? 1 : TAPS;
  if (TAPS != kMaxTaps) taps = TAPS;
  float inv[NT];
  float* st = nullptr;
  int64_t pos = 0;
  int local = 0;
  if (cw != nullptr) {
    const int s = row_seq[t];
    pos = positions[t];
    local = (int)(pos - start_pos[s]);
    st = state + ((size_t)slots[s] * nsub + sub) * keep * W;
  } else {
    taps = 1;     // only the add: tap 0 is this row
  }
#pragma unroll
  for (int k = 0; k < NT; ++k) {
    inv[k] = 0.f;
    if (k < taps && y != nullptr) {
      const Tap tp = tap_of(k, t, local, pos, taps);
      if (tp.kind == 1) {
        const YT* yr = y + tp.at * W;
        const YT* y2r = y2 ? y2 + tp.at * W : nullptr;
        float ss = 0.f;
        for (int c = threadIdx.x; c < W; c += blockDim.x) {
          const float v = DT<YT>::load(yr + c) + (y2r ? DT<YT>::load(y2r + c) : 0.f);
          ss += v * v;
        }
        inv[k] = rsqrtf(rt::block_sum(ss, scratch) / W + eps);
      }
    }
  }
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float acc = 0.f, v0 = 0.f;
    const float nwc = y != nullptr ? nw[c] : 0.f;
#pragma unroll
    for (int k = 0; k < NT; ++k) {
      if (k < taps) {
        const Tap tp = tap_of(k, t, local, pos, taps);
        float v = 0.f;
        if (tp.kind == 1) {
          v = x[tp.at * W + c];
          if (y != nullptr) {
            const float yy = DT<YT>::load(y + tp.at * W + c) + (y2 ? DT<YT>::load(y2 + tp.at * W + c) : 0.f);
            v += yy * inv[k] * nwc;
          }
        } else if (tp.kind == 2) {
          v = st[tp.at * W + c];
        }
        if (k == 0) v0 = v;
        if (cw != nullptr) acc += cw[(size_t)c * taps + (taps - 1 - k)] * v;
      }
    }
    if (y != nullptr) xs[(size_t)t * W + c] = v0;
    if (cw != nullptr) {
      DT<OT>::store(h + (size_t)t * W + c, v0 + acc);
      if (shift_state && taps > 1) {
        // one row per sequence (a decode step): this workgroup is the only reader of the sequence's
        // state, and a lane has read its column's old rows above, so it shifts the column here
        for (int i = 0; i + 2 < taps; ++i)
          st[(size_t)i * W + c] = (pos - (taps - 2 - i) >= 0) ? st[(size_t)(i + 1) * W + c] : 0.f;
        st[(size_t)(taps - 2) * W + c] = v0;
      }
    }
  }
}

// a workgroup per (sequence, 256 channels): the last `keep` rows of the span (columns col_off .. col_off + C
// of x) become the sequence's state; a shorter span keeps the newest old rows
template <typename XT>
__global__ void __launch_bounds__(kThreads) conv_state_kernel(const XT* __restrict__ x, int stride, int col_off, int C,
                                                              float* __restrict__ state, int sub, int nsub, int keep,
                                                              const int* __restrict__ cu_q,
                                                              const int* __restrict__ start_pos,
                                                              const int* __restrict__ slots) {
  const int s = blockIdx.x;
  const int r0 = cu_q[s], n = cu_q[s + 1] - r0;
  if (n <= 0) return;
  float* st = state + ((size_t)slots[s] * nsub + sub) * keep * C;
  const int p0 = start_pos[s];
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c < C) {
    float nv[kMaxTaps];
#pragma unroll
    for (int i = 0; i < kMaxTaps; ++i) {
      nv[i] = 0.f;
      if (i < keep) {
        const int idx = n - keep + i;   // row of this span, or (< 0) a row of the old state
        if (idx >= 0) nv[i] = DT<XT>::load(x + (size_t)(r0 + idx) * stride + col_off + c);
        else if (p0 + idx >= 0) nv[i] = st[(size_t)(keep + idx) * C + c];
      }
    }
#pragma unroll
    for (int i = 0; i < kMaxTaps; ++i)
      if (i < keep) st[(size_t)i * C + c] = nv[i];
  }
}

// dynamic LDS: the biased query row [H * Dk], then the biased key row [G * Dk]
template <typename T>
__global__ void __launch_bounds__(kThreads) qkv_prep_wide_kernel(
    T* __restrict__ qo, const T* __restrict__ proj, int stride, int q_off, int k_off, int v_off, int v_from_k,
    const float* __restrict__ qb, const float* __restrict__ kb, const float* __restrict__ qw,
    const float* __restrict__ kw, const float* __restrict__ freq, int R, float mag, const float* __restrict__ vfreq,
    float eps, const int64_t* __restrict__ positions, T* __restrict__ kc, T* __restrict__ vc,
    const int64_t* __restrict__ slot_mapping, int H, int G, int Dk, int Dv, int BS) {
  extern __shared__ float row[];
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const T* pr = proj + (size_t)t * stride;
  const int nq = H * Dk, nk = G * Dk;
  float* qr = row;
  float* kr = row + nq;
  const float pos = (float)positions[t];
  const int64_t slot = slot_mapping[t];
  const size_t blk = (size_t)(slot / BS);
  const int boff = (int)(slot % BS);
  float ssq = 0.f, ssk = 0.f;
  for (int c = threadIdx.x; c < nq; c += blockDim.x) {
    const float v = DT<T>::load(pr + q_off + c) + (qb ? qb[c] : 0.f);
    qr[c] = v;
    ssq += v * v;
  }
  for (int c = threadIdx.x; c < nk; c += blockDim.x) {
    const float v = DT<T>::load(pr + k_off + c) + (kb ? kb[c] : 0.f);
    kr[c] = v;
    ssk += v * v;
    if (v_from_k) {     // the values are the keys as projected (Dv == Dk)
      const int g = c / Dk, d = c - g * Dk;
      DT<T>::store(vc + ((blk * G + g) * BS + boff) * Dv + d, v);
    }
  }
  const float iq = rsqrtf(rt::block_sum(ssq, scratch) / nq + eps);
  const float ik = rsqrtf(rt::block_sum(ssk, scratch) / nk + eps);
  __syncthreads();
  // every lane owns whole pairs: (i, i + R) for i < R, single entries from 2R on
  const int per = Dk - R;       // work items per head: R pairs + (Dk - 2R) singles
  for (int w = threadIdx.x; w < (H + G) * per; w += blockDim.x) {
    const int hh = w / per, i = w - hh * per;
    const bool isq = hh < H;
    const int head = isq ? hh : hh - H;
    const float* src = (isq ? qr : kr) + head * Dk;
    const float* wt = (isq ? qw : kw) + head * Dk;
    const float nrm = isq ? iq : ik;
    T* dst = isq ? qo + ((size_t)t * H + head) * Dk : kc + ((blk * G + head) * BS + boff) * Dk;
    if (i < R) {
      float sn, cs;
      sincosf(pos * freq[i], &sn, &cs);
      sn *= mag;
      cs *= mag;
      const float u = src[i] * nrm * wt[i], v = src[i + R] * nrm * wt[i + R];
      DT<T>::store(dst + i, u * cs - v * sn);
      DT<T>::store(dst + i + R, v * cs + u * sn);
    } else {
      const int d = i + R;
      DT<T>::store(dst + d, src[d] * nrm * wt[d]);
    }
  }
  if (!v_from_k) {
    const int RV = vfreq ? Dv / 2 : 0;
    const int perv = Dv - RV;
    for (int w = threadIdx.x; w < G * perv; w += blockDim.x) {
      const int g = w / perv, i = w - g * perv;
      const T* src = pr + v_off + g * Dv;
      T* dst = vc + ((blk * G + g) * BS + boff) * Dv;
      if (i < RV) {
        float sn, cs;
        sincosf(pos * vfreq[i], &sn, &cs);
        const float u = DT<T>::load(src + i), v = DT<T>::load(src + i + RV);
        DT<T>::store(dst + i, u * cs - v * sn);
        DT<T>::store(dst + i + RV, v * cs + u * sn);
      } else {
        const int d = i + RV;
        DT<T>::store(dst + d, DT<T>::load(src + d));
      }
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(kThreads) turn_back_kernel(T* __restrict__ out, int out_stride, int out_off,
                                                             const T* __restrict__ o, int H, int E,
                                                             const int64_t* __restrict__ positions,
                                                             const float* __restrict__ vfreq, float scale) {
  const int t = blockIdx.x;
  const float pos = -(float)positions[t];
  const int R = E / 2, per = E - R;
  for (int w = threadIdx.x; w < H * per; w += blockDim.x) {
    const int h = w / per, i = w - h * per;
    const T* src = o + ((size_t)t * H + h) * E;
    T* dst = out + (size_t)t * out_stride + out_off + h * E;
    if (i < R) {
      float sn, cs;
      sincosf(pos * vfreq[i], &sn, &cs);
      const float u = DT<T>::load(src + i), v = DT<T>::load(src + i + R);
      DT<T>::store(dst + i, (u * cs - v * sn) * scale);
      DT<T>::store(dst + i + R, (v * cs + u * sn) * scale);
    } else {
      DT<T>::store(dst + i + R, DT<T>::load(src + i + R) * scale);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(kThreads) silu_cols_kernel(float* __restrict__ out, const T* __restrict__ proj,
                                                             int stride, int off, int n, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const int64_t r = i / n;
  out[i] = silu(DT<T>::load(proj + r * stride + off + (i - r * n)));
}

template <typename T>
__global__ void __launch_bounds__(kThreads) relu2_kernel(T* __restrict__ out, const T* __restrict__ a, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const float v = fmaxf(DT<T>::load(a + i), 0.f);
  DT<T>::store(out + i, v * v);
}

// bf16, a multiple of 8 entries: 16-byte loads and stores
__global__ void __launch_bounds__(kThreads) relu2_8_kernel(uint16_t* __restrict__ out, const uint16_t* __restrict__ a,
                                                           int64_t groups) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= groups) return;
  const rt::short8 v = *reinterpret_cast<const rt::short8*>(a + i * 8);
  rt::short8 o;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const float f = fmaxf(rt::bf2f((uint16_t)v[j]), 0.f);
    o[j] = (short)rt::f2bf(f * f);
  }
  *reinterpret_cast<rt::short8*>(out + i * 8) = o;
}

// out [6][T][A * D] = r, k, v, w, a * u, u; one wave per head
template <typename T>
__global__ void __launch_bounds__(kThreads) removal_prep_kernel(
    float* __restrict__ out, const T* __restrict__ proj, int stride, int r_off, int k_off, int v_off, int a_off,
    const T* __restrict__ lw, const float* __restrict__ w0, const float* __restrict__ ab, int Tn, int A, int D) {
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const T* pr = proj + (size_t)t * stride;
  const size_t n = (size_t)A * D, plane = (size_t)Tn * n;
  const float kdec = -0.60653065971263342f;     // -e^(-1/2)
  for (int a = wave; a < A; a += nw) {
    float ss = 0.f;
    for (int d = lane; d < D; d += 64) {
      const float kv = DT<T>::load(pr + k_off + a * D + d);
      ss += kv * kv;
    }
    const float iu = rsqrtf(rt::wave_sum(ss) + 1e-6f);
    for (int d = lane; d < D; d += 64) {
      const int c = a * D + d;
      float* o = out + (size_t)t * n + c;
      const float kv = DT<T>::load(pr + k_off + c);
      const float u = kv * iu;
      o[0] = DT<T>::load(pr + r_off + c);
      o[plane] = kv;
      o[2 * plane] = DT<T>::load(pr + v_off + c);
      o[3 * plane] = __expf(kdec * sigm(DT<T>::load(lw + (size_t)t * n + c) + w0[c]));
      o[4 * plane] = sigm(DT<T>::load(pr + a_off + c) + ab[c]) * u;
      o[5 * plane] = u;
    }
  }
}

// dynamic LDS: z [C] (convolved, silu), then the unit factors of the G query heads and G key heads
template <typename T>
__global__ void __launch_bounds__(1024) delta_prep_kernel(
    float* __restrict__ five, float* __restrict__ vout, const T* __restrict__ proj, int stride, int q_off, int b_off,
    int a_off, const float* __restrict__ cw, float* __restrict__ state, const float* __restrict__ neg_rate,
    const float* __restrict__ dt_bias, int Tn, int A, int G, int D, int E, int taps, int keep,
    const int* __restrict__ row_seq, const int64_t* __restrict__ positions, const int* __restrict__ start_pos,
    const int* __restrict__ slots, int shift_state) {
  extern __shared__ float z[];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const int C = 2 * G * D + A * E;
  float* unit = z + C;          // [2 * G]
  const int s = row_seq[t];
  const int64_t pos = positions[t];
  const int local = (int)(pos - start_pos[s]);
  float* st = state + (size_t)slots[s] * keep * C;
  for (int c = threadIdx.x; c < C; c += blockDim.x) {
    float acc = 0.f, v0 = 0.f;
    for (int k = 0; k < taps; ++k) {
      const Tap tp = tap_of(k, t, local, pos, taps);
      float v = 0.f;
      if (tp.kind == 1) v = DT<T>::load(proj + tp.at * stride + q_off + c);
      else if (tp.kind == 2) v = st[tp.at * C + c];
      if (k == 0) v0 = v;
      acc += cw[(size_t)c * taps + (taps - 1 - k)] * v;
    }
    z[c] = silu(acc);
    if (shift_state && taps > 1) {
      for (int i = 0; i + 2 < taps; ++i)
        st[(size_t)i * C + c] = (pos - (taps - 2 - i) >= 0) ? st[(size_t)(i + 1) * C + c] : 0.f;
      st[(size_t)(taps - 2) * C + c] = v0;
    }
  }
  __syncthreads();
  for (int j = wave; j < 2 * G; j += nw) {     // q heads, then k heads
    float ss = 0.f;
    for (int d = lane; d < D; d += 64) ss += z[j * D + d] * z[j * D + d];
    const float iv = rsqrtf(rt::wave_sum(ss) + 1e-6f);
    if (lane == 0) unit[j] = iv;
  }
  __syncthreads();
  const size_t n = (size_t)A * D, plane = (size_t)Tn * n;
  const int rep = A / G;
  const float qs = rsqrtf((float)D);
  const T* pr = proj + (size_t)t * stride;
  for (int a = wave; a < A; a += nw) {
    const int g = a / rep;
    const float beta = sigm(DT<T>::load(pr + b_off + a));
    const float xa = DT<T>::load(pr + a_off + a) + dt_bias[a];
    const float sp = xa > 20.f ? xa : log1pf(__expf(xa));
    const float gd = __expf(neg_rate[a] * sp);
    for (int d = lane; d < D; d += 64) {
      float* o = five + (size_t)t * n + a * D + d;
      const float qv = z[g * D + d] * unit[g] * qs;
      const float kv = z[(G + g) * D + d] * unit[G + g];
      o[0] = qv;
      o[plane] = beta * kv;
      o[2 * plane] = gd;
      o[3 * plane] = gd * beta * kv;
      o[4 * plane] = kv;
    }
  }
  for (int c = threadIdx.x; c < A * E; c += blockDim.x) vout[(size_t)t * A * E + c] = z[2 * G * D + c];
}

// out [T][3 n + nv] = q * q_scale, k, decay (n = heads * dim columns each), v; a2 [rank][n] is the second
// factor of the decay's low-rank path, read once for ROWS rows. dynamic LDS: the rows' rank inputs.
// decay = sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau)
template <typename T, int ROWS>
__global__ void __launch_bounds__(1024) gla_prep_kernel(float* __restrict__ out, const T* __restrict__ proj, int stride,
                                                        int q_off, int k_off, int v_off, int a_off, int rank,
                                                        const float* __restrict__ a2, const float* __restrict__ ab,
                                                        float q_scale, float inv_tau, int Tn, int n, int nv) {
  extern __shared__ float low[];        // [ROWS][rank]
  const int t0 = blockIdx.x * ROWS;
  const int rows = min(ROWS, Tn - t0);
  for (int i = threadIdx.x; i < ROWS * rank; i += blockDim.x) {
    const int r = i / rank;
    low[i] = r < rows ? DT<T>::load(proj + (size_t)(t0 + r) * stride + a_off + (i - r * rank)) : 0.f;
  }
  __syncthreads();
  const size_t os = (size_t)3 * n + nv;
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    float z[ROWS];
    const float bc = ab[c];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) z[r] = bc;
#pragma unroll 4
    for (int j = 0; j < rank; ++j) {
      const float wv = a2[(size_t)j * n + c];
#pragma unroll
      for (int r = 0; r < ROWS; ++r) z[r] += wv * low[r * rank + j];
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
      if (r < rows) {
        const T* pr = proj + (size_t)(t0 + r) * stride;
        float* o = out + (size_t)(t0 + r) * os;
        o[c] = DT<T>::load(pr + q_off + c) * q_scale;
        o[n + c] = DT<T>::load(pr + k_off + c);
        o[2 * (size_t)n + c] = expf(-(fmaxf(-z[r], 0.f) + log1pf(expf(-fabsf(z[r])))) * inv_tau);
      }
  }
  for (int r = 0; r < rows; ++r)
    for (int c = threadIdx.x; c < nv; c += blockDim.x)
      out[(size_t)(t0 + r) * os + 3 * (size_t)n + c] = DT<T>::load(proj + (size_t)(t0 + r) * stride + v_off + c);
}

RT_DEVICE float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// out [4][T][n] = q, beta k, g, g k per value head (n = A * D), vout [T][A * E]; a2 [rank][n]. A workgroup
// takes ROWS rows of one query / key head and its value heads (no norm or state crosses heads): all its
// convolution inputs and low-rank terms are in flight together, which is what few rows wait for, and ROWS
// rows share a pass over a2. dynamic LDS: low [ROWS][rank], part [parts][ROWS][m] (m = rep * D decay
// columns, the rank split over `parts` groups of lanes), z [ROWS][Cg], unit factors [ROWS][2].
// TAPS: the taps as a compile-time number, or 0 for any number
template <typename T, int ROWS, int TAPS>
__global__ void __launch_bounds__(kThreads) channel_delta_kernel(
    float* __restrict__ out, float* __restrict__ vout, const T* __restrict__ proj, int stride, int q_off, int b_off,
    int a_off, int rank, const float* __restrict__ a2, const float* __restrict__ cw, float* __restrict__ state,
    const float* __restrict__ neg_rate, const float* __restrict__ dt_bias, int Tn, int A, int G, int D, int E, int taps,
    int keep, const int* __restrict__ row_seq, const int64_t* __restrict__ positions, const int* __restrict__ start_pos,
    const int* __restrict__ slots, int shift_state, int parts) {
  extern __shared__ float lds[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int n = A * D, C = 2 * G * D + A * E, rep = A / G, g = blockIdx.y;
  const int m = rep * D, Cg = 2 * D + rep * E;
  float* low = lds;
  float* part = low + ROWS * rank;
  float* z = part + parts * ROWS * m;
  float* unit = z + ROWS * Cg;
  const int t0 = blockIdx.x * ROWS;
  const int rows = min(ROWS, Tn - t0);
  for (int i = threadIdx.x; i < ROWS * rank; i += kThreads) {
    const int r = i / rank;
    low[i] = r < rows ? DT<T>::load(proj + (size_t)(t0 + r) * stride + a_off + (i - r * rank)) : 0.f;
  }
  // rows of one span with all their predecessors in this batch: every row is read once, without branches
  const bool inner = TAPS > 0 && rows == ROWS && row_seq[t0] == row_seq[t0 + ROWS - 1] &&
                     positions[t0] - start_pos[row_seq[t0]] >= TAPS - 1;
  for (int c = threadIdx.x; c < Cg; c += kThreads) {
    // channel of the projection: this head's q, its k, its value heads' v
    const int ch = c < D ? g * D + c : c < 2 * D ? G * D + g * D + (c - D) : 2 * G * D + g * rep * E + (c - 2 * D);
    if (TAPS > 0 && inner) {
      constexpr int NX = TAPS > 0 ? TAPS : 1;
      float x[ROWS + NX - 1], wk[NX];
#pragma unroll
      for (int i = 0; i < ROWS + NX - 1; ++i) x[i] = DT<T>::load(proj + (size_t)(t0 - (NX - 1) + i) * stride + q_off + ch);
#pragma unroll
      for (int k = 0; k < NX; ++k) wk[k] = cw[(size_t)ch * NX + k];
#pragma unroll
      for (int r = 0; r < ROWS; ++r) {
        float acc = 0.f;
#pragma unroll
        for (int k = 0; k < NX; ++k) acc += wk[NX - 1 - k] * x[r + NX - 1 - k];
        const float sv = silu(acc);
        z[r * Cg + c] = sv;
        if (c >= 2 * D) vout[(size_t)(t0 + r) * A * E + g * rep * E + (c - 2 * D)] = sv;
      }
      continue;
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      if (r >= rows) break;
      const int t = t0 + r, s = row_seq[t];
      const int64_t pos = positions[t];
      const int local = (int)(pos - start_pos[s]);
      float* st = state + (size_t)slots[s] * keep * C + ch;
      float acc = 0.f, v0 = 0.f;
      for (int k = 0; k < taps; ++k) {
        const Tap tp = tap_of(k, t, local, pos, taps);
        float v = 0.f;
        if (tp.kind == 1) v = DT<T>::load(proj + tp.at * stride + q_off + ch);
        else if (tp.kind == 2) v = st[tp.at * C];
        if (k == 0) v0 = v;
        acc += cw[(size_t)ch * taps + (taps - 1 - k)] * v;
      }
      const float sv = silu(acc);
      z[r * Cg + c] = sv;
      if (c >= 2 * D) vout[(size_t)t * A * E + g * rep * E + (c - 2 * D)] = sv;
      if (shift_state && taps > 1) {
        for (int i = 0; i + 2 < taps; ++i)
          st[(size_t)i * C] = (pos - (taps - 2 - i) >= 0) ? st[(size_t)(i + 1) * C] : 0.f;
        st[(size_t)(taps - 2) * C] = v0;
      }
    }
  }
  __syncthreads();
  for (int w = threadIdx.x; w < parts * m; w += kThreads) {
    const int pt = w / m, c = w - pt * m;
    const int j0 = rank * pt / parts, j1 = rank * (pt + 1) / parts;
    const float* col = a2 + g * m + c;
    float x[ROWS];
#pragma unroll
    for (int r = 0; r < ROWS; ++r) x[r] = 0.f;
#pragma unroll 16
    for (int j = j0; j < j1; ++j) {
      const float wv = col[(size_t)j * n];
#pragma unroll
      for (int r = 0; r < ROWS; ++r) x[r] += wv * low[r * rank + j];
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) part[(pt * ROWS + r) * m + c] = x[r];
  }
  for (int j = wave; j < 2 * rows; j += kThreads / 64) {      // (row, q or k)
    const float* zz = z + (j >> 1) * Cg + (j & 1) * D;
    float ss = 0.f;
    for (int d = lane; d < D; d += 64) ss += zz[d] * zz[d];
    const float iv = 1.0f / sqrtf(rt::wave_sum(ss) + 1e-6f);
    if (lane == 0) unit[j] = iv;
  }
  __syncthreads();
  const size_t plane = (size_t)Tn * n;
  const float qs = 1.0f / sqrtf((float)D);
  for (int w = threadIdx.x; w < rows * m; w += kThreads) {
    const int r = w / m, c = w - r * m;
    const int a = g * rep + c / D, d = c % D;
    const T* pr = proj + (size_t)(t0 + r) * stride;
    float x = dt_bias[g * m + c];
    for (int pt = 0; pt < parts; ++pt) x += part[(pt * ROWS + r) * m + c];
    const float gd = expf(neg_rate[a] * softplus(x));
    const float beta = 1.0f / (1.0f + expf(-DT<T>::load(pr + b_off + a)));
    const float kv = z[r * Cg + D + d] * unit[2 * r + 1];
    float* o = out + (size_t)(t0 + r) * n + g * m + c;
    o[0] = z[r * Cg + d] * unit[2 * r] * qs;
    o[plane] = beta * kv;
    o[2 * plane] = gd;
    o[3 * plane] = gd * kv;
  }
}

// the gates of one (token, head): the capped log input gate and the log of the capped forget gate
RT_DEVICE void memory_gate(float pi, float pf, float cap, float& gi, float& gf) {
  gi = cap * tanhf(pi / cap);
  gf = -softplus(-cap * tanhf(pf / cap));
}

// gates [3][T][A] = exp(f_t + m_(t-1) - m_t), exp(i_t - m_t), exp(-m_t) with m_t = max(f_t + m_(t-1), i_t), m
// from gmax[slot] (0 at position 0). A workgroup per (sequence, head), 64 tokens per wave: a scan over the
// maps m -> max(m + a, b), of which two in a row are (a1 + a2, max(b1 + a2, b2)), inside every wave, then
// over the waves' whole maps.
template <typename T>
__global__ void __launch_bounds__(1024) memory_gates_kernel(float* __restrict__ gates, const T* __restrict__ proj, int stride,
                                                            int i_off, int f_off, const float* __restrict__ ib,
                                                            const float* __restrict__ fb, float cap, float* __restrict__ gmax,
                                                            const int* __restrict__ cu_q, const int* __restrict__ start_pos,
                                                            const int* __restrict__ slots, int Tn, int A) {
  __shared__ float wa[2][16], wb[2][16];      // every wave's whole map, two sets in turn
  const int s = blockIdx.x, a = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const int r0 = cu_q[s], n = cu_q[s + 1] - r0;
  if (n <= 0) return;
  float* mp = gmax + (size_t)slots[s] * A + a;
  float m = start_pos[s] > 0 ? *mp : 0.f;
  const size_t plane = (size_t)Tn * A;
  const float bi = ib[a], bf = fb[a];
  const T* pa0 = proj + (size_t)r0 * stride + a;
  float ni = DT<T>::load(pa0 + (size_t)min((int)threadIdx.x, n - 1) * stride + i_off);      // one round ahead
  float nf = DT<T>::load(pa0 + (size_t)min((int)threadIdx.x, n - 1) * stride + f_off);
  int set = 0;
  for (int c0 = 0; c0 < n; c0 += (int)blockDim.x, set ^= 1) {
    const int t = c0 + threadIdx.x;
    float gi, gf;
    memory_gate(ni + bi, nf + bf, cap, gi, gf);
    if (t >= n) {       // the identity
      gi = -INFINITY;
      gf = 0.f;
    }
    const size_t nt = (size_t)min(t + (int)blockDim.x, n - 1) * stride;
    ni = DT<T>::load(pa0 + nt + i_off);
    nf = DT<T>::load(pa0 + nt + f_off);
    float sa = gf, sb = gi;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float pa = __shfl_up(sa, o, 64), pb = __shfl_up(sb, o, 64);
      if (lane >= o) {
        sb = fmaxf(pb + sa, sb);
        sa = pa + sa;
      }
    }
    if (lane == 63) {
      wa[set][wave] = sa;
      wb[set][wave] = sb;
    }
    __syncthreads();      // (a set is written again two rounds later, past the next round's barrier)
    float mw = m;         // the maximum ahead of this wave's tokens
    for (int w = 0; w < nw; ++w) {
      if (w == wave) mw = m;
      m = fmaxf(m + wa[set][w], wb[set][w]);
    }
    const float mt = fmaxf(mw + sa, sb);
    float before = __shfl_up(mt, 1, 64);
    if (lane == 0) before = mw;
    if (t < n) {
      float* g = gates + (size_t)(r0 + t) * A + a;
      g[0] = expf(gf + before - mt);
      g[plane] = expf(gi - mt);
      g[2 * plane] = expf(-mt);
      if (t == n - 1) *mp = mt;
    }
  }
}

// out [T][2 n + A (E + 1)] = q * q_scale, weight * k (n = A * D columns each), per head v and a one.
// gates as written by memory_gates; STEP: one row per sequence, the gates are formed here from gmax
template <typename T, bool STEP>
__global__ void __launch_bounds__(1024) memory_prep_kernel(float* __restrict__ out, float* __restrict__ gates,
                                                           const T* __restrict__ proj, int stride, int q_off, int k_off,
                                                           int v_off, int i_off, int f_off, const float* __restrict__ ib,
                                                           const float* __restrict__ fb, float cap,
                                                           float* __restrict__ gmax, const int* __restrict__ start_pos,
                                                           const int* __restrict__ slots, float q_scale, int Tn, int A, int D,
                                                           int E) {
  extern __shared__ float lds[];      // [A]: weights
  const int t = blockIdx.x;
  const T* pr = proj + (size_t)t * stride;
  const size_t plane = (size_t)Tn * A;
  const int n = A * D;
  for (int a = threadIdx.x; a < A; a += blockDim.x) {
    float* g = gates + (size_t)t * A + a;
    if (STEP) {
      float* mp = gmax + (size_t)slots[t] * A + a;
      const float m = start_pos[t] > 0 ? *mp : 0.f;
      float gi, gf;
      memory_gate(DT<T>::load(pr + i_off + a) + ib[a], DT<T>::load(pr + f_off + a) + fb[a], cap, gi, gf);
      const float mt = fmaxf(gf + m, gi);
      *mp = mt;
      lds[a] = expf(gi - mt);
      g[0] = expf(gf + m - mt);
      g[2 * plane] = expf(-mt);
    } else {
      lds[a] = g[plane];
    }
  }
  __syncthreads();
  float* o = out + (size_t)t * (2 * (size_t)n + (size_t)A * (E + 1));
  for (int c = threadIdx.x; c < n; c += blockDim.x) {
    const int a = c / D;
    o[c] = DT<T>::load(pr + q_off + c) * q_scale;
    o[n + c] = DT<T>::load(pr + k_off + c) * lds[a];
  }
  for (int c = threadIdx.x; c < A * (E + 1); c += blockDim.x) {
    const int a = c / (E + 1), e = c - a * (E + 1);
    o[2 * (size_t)n + c] = e < E ? DT<T>::load(pr + v_off + a * E + e) : 1.0f;
  }
}

// o [T, C] fp32: segments of `span` entries are divided by their RMS; wmod = entries of the weight.
// floors [T, C / span]: o has one more entry per segment, n . q, and a segment is divided by
// max(|n . q|, floor) + 1e-6 first.
template <typename OT, typename GT>
__global__ void __launch_bounds__(1024) head_norm_gate_kernel(
    OT* __restrict__ out, int out_stride, int out_off, const float* __restrict__ o, const float* __restrict__ w, int wmod,
    int span, const GT* __restrict__ gate, int gate_stride, int gate_off, int act, float eps, float scale, int C,
    const float* __restrict__ floors) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const int heads = C / span, seg = floors ? span + 1 : span;
  const float* orow = o + (size_t)t * heads * seg;
  const GT* grow = gate + (size_t)t * gate_stride + gate_off;
  OT* dst = out + (size_t)t * out_stride + out_off;
  if (span == C && !floors) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < C; c += blockDim.x) ss += orow[c] * orow[c];
    const float iv = rsqrtf(rt::block_sum(ss, scratch) / C + eps);
    for (int c = threadIdx.x; c < C; c += blockDim.x) {
      const float g = DT<GT>::load(grow + c);
      DT<OT>::store(dst + c, orow[c] * iv * w[c % wmod] * (act ? silu(g) : sigm(g)) * scale);
    }
    return;
  }
  for (int h = wave; h < heads; h += nw) {
    const float* os = orow + h * seg;
    const float den = floors ? 1.0f / (fmaxf(fabsf(os[span]), floors[(size_t)t * heads + h]) + 1e-6f) : 1.0f;
    float ss = 0.f;
    for (int d = lane; d < span; d += 64) ss += os[d] * os[d];
    const float iv = den * rsqrtf(rt::wave_sum(ss) * den * den / span + eps);
    for (int d = lane; d < span; d += 64) {
      const int c = h * span + d;
      const float g = DT<GT>::load(grow + c);
      DT<OT>::store(dst + c, os[d] * iv * w[c % wmod] * (act ? silu(g) : sigm(g)) * scale);
    }
  }
}

}  // namespace

void launch_canon_add(void* h, float* xs, const float* x, const void* y, const void* y2, const float* nw, float eps,
                      const float* cw, float* state, int sub, int nsub, const int* row_seq, const int64_t* positions,
                      const int* start_pos, const int* slots, int T, int W, int taps, int keep, bool out_bf, bool y_bf,
                      bool shift_state, hipStream_t stream) {
  if (T <= 0) return;
  // about one entry per lane (64 .. 1024 lanes): a row's loads leave together, which is what a
  // decode step of a few rows waits for
  const int th = W >= 1024 ? 1024 : W <= 64 ? 64 : (W + 63) / 64 * 64;
#define RT_CA2(OT, YT, TP)                                                                                             \
  canon_add_kernel<OT, YT, TP><<<T, th, 0, stream>>>((OT*)h, xs, x, (const YT*)y, (const YT*)y2, nw, eps, cw,     \
                                                           state, sub, nsub, row_seq, positions, start_pos, slots, W,    \
                                                           taps, keep, shift_state ? 1 : 0)
#define RT_CA(OT, YT)                                                                                                  \
  do {                                                                                                                 \
    const int tp = cw == nullptr ? 0 : taps;                                                                           \
    if (tp == 0) RT_CA2(OT, YT, 0); else if (tp == 1) RT_CA2(OT, YT, 1); else if (tp == 2) RT_CA2(OT, YT, 2);          \
    else if (tp == 3) RT_CA2(OT, YT, 3); else if (tp == 4) RT_CA2(OT, YT, 4); else RT_CA2(OT, YT, kMaxTaps);           \
  } while (0)
  if (out_bf) {
    if (y_bf) RT_CA(uint16_t, uint16_t); else RT_CA(uint16_t, float);
  } else {
    if (y_bf) RT_CA(float, uint16_t); else RT_CA(float, float);
  }
#undef RT_CA
#undef RT_CA2
}

void launch_conv_state(const void* x, int stride, int col_off, int C, float* state, int sub, int nsub, int keep,
                       const int* cu_q, const int* start_pos, const int* slots, int S, bool bf, hipStream_t stream) {
  if (S <= 0) return;
  const dim3 grid(S, (C + kThreads - 1) / kThreads);
  if (bf) conv_state_kernel<uint16_t><<<grid, kThreads, 0, stream>>>((const uint16_t*)x, stride, col_off, C, state, sub, nsub,
                                                                   keep, cu_q, start_pos, slots);
  else conv_state_kernel<float><<<grid, kThreads, 0, stream>>>((const float*)x, stride, col_off, C, state, sub, nsub, keep,
                                                            cu_q, start_pos, slots);
}

int launch_qkv_prep_wide(void* q, const void* proj, int stride, int q_off, int k_off, int v_off, bool v_from_k,
                         const float* qb, const float* kb, const float* qw, const float* kw, const float* freq, int R,
                         float mag, const float* vfreq, float eps, const int64_t* positions, void* kc, void* vc,
                         const int64_t* slot_mapping, int T, int H, int G, int Dk, int Dv, int BS, bool bf,
                         hipStream_t stream) {
  if (T <= 0) return 0;
  const size_t shm = sizeof(float) * (size_t)(H + G) * Dk;
  if (shm > 150 * 1024) return -1;
#define RT_QW(TT)                                                                                                      \
  do {                                                                                                                 \
    auto kern = qkv_prep_wide_kernel<TT>;                                                                              \
    if (shm > 48 * 1024 &&                                                                                             \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm) != hipSuccess)    \
      return -2;                                                                                                       \
    kern<<<T, kThreads, shm, stream>>>((TT*)q, (const TT*)proj, stride, q_off, k_off, v_off, v_from_k ? 1 : 0, qb, kb,  \
                                       qw, kw, freq, R, mag, vfreq, eps, positions, (TT*)kc, (TT*)vc, slot_mapping, H,  \
                                       G, Dk, Dv, BS);                                                                 \
  } while (0)
  if (bf) RT_QW(uint16_t); else RT_QW(float);
#undef RT_QW
  return 0;
}

void launch_turn_back(void* out, int out_stride, int out_off, const void* o, int T, int H, int E,
                      const int64_t* positions, const float* vfreq, float scale, bool bf, hipStream_t stream) {
  if (T <= 0) return;
  if (bf) turn_back_kernel<uint16_t><<<T, kThreads, 0, stream>>>((uint16_t*)out, out_stride, out_off, (const uint16_t*)o, H,
                                                                  E, positions, vfreq, scale);
  else turn_back_kernel<float><<<T, kThreads, 0, stream>>>((float*)out, out_stride, out_off, (const float*)o, H, E,
                                                           positions, vfreq, scale);
}

void launch_silu_cols(float* out, const void* proj, int stride, int off, int n, int T, bool bf, hipStream_t stream) {
  const int64_t total = (int64_t)T * n;
  if (total <= 0) return;
  const int blocks = (int)((total + kThreads - 1) / kThreads);
  if (bf) silu_cols_kernel<uint16_t><<<blocks, kThreads, 0, stream>>>(out, (const uint16_t*)proj, stride, off, n, total);
  else silu_cols_kernel<float><<<blocks, kThreads, 0, stream>>>(out, (const float*)proj, stride, off, n, total);
}

void launch_relu2(void* out, const void* a, int64_t total, bool bf, hipStream_t stream) {
  if (total <= 0) return;
  if (bf && total % 8 == 0 && ((reinterpret_cast<uintptr_t>(a) | reinterpret_cast<uintptr_t>(out)) & 15) == 0) {
    const int64_t groups = total / 8;
    relu2_8_kernel<<<(int)((groups + kThreads - 1) / kThreads), kThreads, 0, stream>>>((uint16_t*)out, (const uint16_t*)a,
                                                                                      groups);
    return;
  }
  const int blocks = (int)((total + kThreads - 1) / kThreads);
  if (bf) relu2_kernel<uint16_t><<<blocks, kThreads, 0, stream>>>((uint16_t*)out, (const uint16_t*)a, total);
  else relu2_kernel<float><<<blocks, kThreads, 0, stream>>>((float*)out, (const float*)a, total);
}

void launch_removal_prep(float* out, const void* proj, int stride, int r_off, int k_off, int v_off, int a_off,
                         const void* lw, const float* w0, const float* ab, int T, int A, int D, bool bf,
                         hipStream_t stream) {
  if (T <= 0) return;
  if (bf) removal_prep_kernel<uint16_t><<<T, kThreads, 0, stream>>>(out, (const uint16_t*)proj, stride, r_off, k_off, v_off,
                                                                     a_off, (const uint16_t*)lw, w0, ab, T, A, D);
  else removal_prep_kernel<float><<<T, kThreads, 0, stream>>>(out, (const float*)proj, stride, r_off, k_off, v_off, a_off,
                                                              (const float*)lw, w0, ab, T, A, D);
}

int launch_delta_prep(float* five, float* vout, const void* proj, int stride, int q_off, int b_off, int a_off,
                      const float* cw, float* state, const float* neg_rate, const float* dt_bias, int T, int A, int G,
                      int D, int E, int taps, int keep, const int* row_seq, const int64_t* positions,
                      const int* start_pos, const int* slots, bool shift_state, bool bf, hipStream_t stream) {
  if (T <= 0) return 0;
  const size_t shm = sizeof(float) * ((size_t)2 * G * D + (size_t)A * E + 2 * G);
  if (shm > 150 * 1024 || taps > kMaxTaps) return -1;
  const int C = 2 * G * D + A * E;
  const int th = C >= 1024 ? 1024 : C <= 256 ? 256 : (C + 63) / 64 * 64;
#define RT_DP(TT)                                                                                                      \
  do {                                                                                                                 \
    auto kern = delta_prep_kernel<TT>;                                                                                 \
    if (shm > 48 * 1024 &&                                                                                             \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm) != hipSuccess)    \
      return -2;                                                                                                       \
    kern<<<T, th, shm, stream>>>(five, vout, (const TT*)proj, stride, q_off, b_off, a_off, cw, state, neg_rate,         \
                                       dt_bias, T, A, G, D, E, taps, keep, row_seq, positions, start_pos, slots,       \
                                       shift_state ? 1 : 0);                                                           \
  } while (0)
  if (bf) RT_DP(uint16_t); else RT_DP(float);
#undef RT_DP
  return 0;
}

int launch_gla_prep(float* out, const void* proj, int stride, int q_off, int k_off, int v_off, int a_off, int rank,
                    const float* a2, const float* ab, float q_scale, float inv_tau, int T, int n, int nv, bool bf,
                    hipStream_t stream) {
  if (T <= 0) return 0;
  const int rows = T >= 256 ? 4 : 1;      // few rows: one workgroup each; many: the low-rank factor is read once for four
  const size_t shm = sizeof(float) * (size_t)rows * rank;
  if (shm > 48 * 1024) return -1;
  const int m = n > nv ? n : nv;
  const int th = m >= 1024 ? 1024 : m <= 64 ? 64 : (m + 63) / 64 * 64;
#define RT_GP(TT, R)                                                                                                   \
  gla_prep_kernel<TT, R><<<(T + R - 1) / R, th, shm, stream>>>(out, (const TT*)proj, stride, q_off, k_off, v_off, a_off, \
                                                               rank, a2, ab, q_scale, inv_tau, T, n, nv)
  if (bf) {
    if (rows == 4) RT_GP(uint16_t, 4); else RT_GP(uint16_t, 1);
  } else {
    if (rows == 4) RT_GP(float, 4); else RT_GP(float, 1);
  }
#undef RT_GP
  return 0;
}

int launch_channel_delta(float* out, float* vout, const void* proj, int stride, int q_off, int b_off, int a_off, int rank,
                         const float* a2, const float* cw, float* state, const float* neg_rate, const float* dt_bias, int T,
                         int A, int G, int D, int E, int taps, int keep, const int* row_seq, const int64_t* positions,
                         const int* start_pos, const int* slots, bool shift_state, bool bf, hipStream_t stream) {
  if (T <= 0) return 0;
  if (taps > kMaxTaps) return -1;
  const int rep = A / G, m = rep * D, Cg = 2 * D + rep * E;
  const int parts = m >= kThreads ? 1 : kThreads / m < rank ? kThreads / m : rank;
  auto lds_of = [&](int rows) { return sizeof(float) * (size_t)rows * (rank + parts * m + Cg + 2); };
  const int rows = T >= 256 && lds_of(4) <= 64 * 1024 ? 4 : 1;    // many rows: the low-rank factor is read once for four
  const size_t shm = lds_of(rows);
  if (shm > 150 * 1024) return -1;
#define RT_CD(TT, R)                                                                                                   \
  do {                                                                                                                 \
    auto kern = R == 4 && taps == 4 ? channel_delta_kernel<TT, R, 4> : R == 4 && taps == 3                             \
                    ? channel_delta_kernel<TT, R, 3> : R == 4 && taps == 2 ? channel_delta_kernel<TT, R, 2>            \
                                                                           : channel_delta_kernel<TT, R, 0>;           \
    if (shm > 48 * 1024 &&                                                                                             \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shm) != hipSuccess)    \
      return -2;                                                                                                       \
    kern<<<dim3((T + R - 1) / R, G), kThreads, shm, stream>>>(out, vout, (const TT*)proj, stride, q_off, b_off, a_off, \
                                                              rank, a2, cw, state, neg_rate, dt_bias, T, A, G, D, E,   \
                                                              taps, keep, row_seq, positions, start_pos, slots,        \
                                                              shift_state ? 1 : 0, parts);                             \
  } while (0)
  if (bf) {
    if (rows == 4) RT_CD(uint16_t, 4); else RT_CD(uint16_t, 1);
  } else {
    if (rows == 4) RT_CD(float, 4); else RT_CD(float, 1);
  }
#undef RT_CD
  return 0;
}

int launch_memory_prep(float* out, float* gates, const void* proj, int stride, int q_off, int k_off, int v_off, int i_off,
                       int f_off, const float* ib, const float* fb, float cap, float* gmax, const int* cu_q,
                       const int* start_pos, const int* slots, float q_scale, int S, int T, int A, int D, int E, bool step,
                       bool bf, hipStream_t stream) {
  if (T <= 0 || S <= 0) return 0;
  const size_t shm = sizeof(float) * (size_t)A;
  if (shm > 48 * 1024) return -1;
  const int m = A * (D > E + 1 ? D : E + 1);
  const int gth = T >= 1024 ? 1024 : (T + 63) / 64 * 64;
  const int th = m >= 1024 ? 1024 : m <= 64 ? 64 : (m + 63) / 64 * 64;
#define RT_MP(TT)                                                                                                      \
  do {                                                                                                                 \
    if (!step)                                                                                                         \
      memory_gates_kernel<TT><<<dim3(S, A), gth, 0, stream>>>(gates, (const TT*)proj, stride, i_off, f_off, ib, fb, cap, \
                                                             gmax, cu_q, start_pos, slots, T, A);                      \
    if (step) memory_prep_kernel<TT, true><<<T, th, shm, stream>>>(out, gates, (const TT*)proj, stride, q_off, k_off,  \
                                                                   v_off, i_off, f_off, ib, fb, cap, gmax, start_pos,  \
                                                                   slots, q_scale, T, A, D, E);                        \
    else memory_prep_kernel<TT, false><<<T, th, shm, stream>>>(out, gates, (const TT*)proj, stride, q_off, k_off,      \
                                                               v_off, i_off, f_off, ib, fb, cap, gmax, start_pos,      \
                                                               slots, q_scale, T, A, D, E);                            \
  } while (0)
  if (bf) RT_MP(uint16_t); else RT_MP(float);
#undef RT_MP
  return 0;
}

void launch_head_norm_gate(void* out, int out_stride, int out_off, const float* o, const float* w, int wmod, int span,
                           const void* gate, int gate_stride, int gate_off, int act, float eps, float scale, int T, int C,
                           const float* floors, bool out_bf, bool gate_bf, hipStream_t stream) {
  if (T <= 0) return;
  // a wave per head, up to 16 waves
  const int th = span == C && !floors ? kThreads : C / span >= 16 ? 1024 : C / span * 64;
#define RT_HN(OT, GT)                                                                                                  \
  head_norm_gate_kernel<OT, GT><<<T, th, 0, stream>>>((OT*)out, out_stride, out_off, o, w, wmod, span,           \
                                                            (const GT*)gate, gate_stride, gate_off, act, eps, scale, C, floors)
  if (out_bf) {
    if (gate_bf) RT_HN(uint16_t, uint16_t); else RT_HN(uint16_t, float);
  } else {
    if (gate_bf) RT_HN(float, uint16_t); else RT_HN(float, float);
  }
#undef RT_HN
}
