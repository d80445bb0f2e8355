// Optional arguments of launchers with many of them (shared by the kernels and the bindings).
#pragma once

// qk_prep: what a projection may get ahead of the norm and the cache
struct QkExtra {
  int halves = 0;                  // rotation pairs (i, i + dims / 2) instead of (2i, 2i + 1)
  const float* q_b = nullptr;      // biases [heads * dim], [kv_heads * dim], [kv_heads * vdim]
  const float* k_b = nullptr;
  const float* v_b = nullptr;
  const void* mix = nullptr;       // value <- (1 - mix_w) value + mix_w (mix[t, g * vdim + d] + mix_b)
  int mix_stride = 0;
  const float* mix_b = nullptr;
  float mix_w = 0.f;
};

// attention: which keys a row sees and what else joins its softmax
struct AttnMask {
  int window = 0;                  // > 0: i - j < window ...
  int keep = 0;                    // ... or j < keep
  int chunk = 0;                   // > 0: j / chunk == i / chunk (with no window)
  const float* sinks = nullptr;    // [heads]: exp(sink) joins the denominator
};

#ifdef __HIPCC__
// oldest key of row position i's own range (keys ahead of it are seen only below `keep`)
__host__ __device__ __forceinline__ int mask_low(const AttnMask& m, int i) {
  if (m.window > 0) return i - m.window + 1 > 0 ? i - m.window + 1 : 0;
  if (m.chunk > 0) return i / m.chunk * m.chunk;
  return 0;
}
__host__ __device__ __forceinline__ bool mask_sees(const AttnMask& m, int low, int i, int j) {
  return j <= i && (j >= low || j < m.keep);
}
// Key tiles of `KT` keys that rows from position `first` up may see: tiles 0 .. kept - 1 (the kept
// first keys), then tiles t0 .. ntile - 1; returns their number, tile_at(v) names the v-th.
struct TileRange {
  int kept, t0, n;
  __host__ __device__ __forceinline__ int at(int v) const { return v < kept ? v : t0 + (v - kept); }
};
__host__ __device__ __forceinline__ TileRange mask_tiles(const AttnMask& m, int first, int kend, int KT) {
  TileRange r;
  r.t0 = mask_low(m, first) / KT;
  const int k = (m.keep + KT - 1) / KT;
  r.kept = k < r.t0 ? k : r.t0;
  r.n = r.kept + (kend + KT - 1) / KT - r.t0;
  return r;
}
#endif
