// A gated linear recurrence with one state element a channel (a real-gated linear recurrent unit): what stands between a
// short convolution's output u and the output projection.
//
//   the C channels are `blocks` equal parts of n channels; for channel c of part b
//   r = sigmoid(Wr[b] u_b + br),  i = sigmoid(Wi[b] u_b + bi)          (Wr[b], Wi[b]: n x n)
//   la = decay[c] r   (decay[c] = -8 softplus(lam[c]), made by the caller),   a = exp(la)
//   S_t = a S_(t-1) + sqrt(1 - a^2) i u,   1 - a^2 = -expm1(2 la);      out = S_t gelu_tanh(y)
//
// A request's state slot holds, per channel, S and behind it the last `hist` inputs of the convolution (float32
// [slots, C, 1 + hist]).  The matrices come in the storage type, laid out [blocks, inner, output]
// (neighbouring threads read neighbouring outputs) or, for the matrix cores, [blocks, output, inner].  Everything behind
// the convolution is float32 whatever the storage type; what a thread sums runs in an order that depends on n alone.
//
//   lru_gates_kernel          la and the addend of every token and channel, any sizes
//   lru_scan_kernel           the walk from the slot's state, a thread a channel
//   lru_step_kernel           one token a sequence: convolution, gates, walk and output in one launch
//   lru_gates_chunk_kernel    bfloat16, many tokens: the gates on the matrix cores for a chunk of 64 tokens, and the chunk's walk
//                             from a state of zero: S from zero and the sum of la up to every token, and at the chunk's end
//   lru_combine_kernel        the walk over a sequence's chunks: the state in front of each, and the slot's final state
//   lru_chunk_out_kernel      S_t = (S from zero) + exp(sum of la) (state in front of the chunk), times gelu_tanh(y)
#include "common.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

#define LRU_MAX_TAPS 16
#define LRU_SLICES 8
#define LRU_TILE 64
#define LRU_CHUNK 64
#define LRU_TB 16
#define LRU_MAX_N 8192       // channels of a part (its u is kept in LDS)

__device__ __forceinline__ void lru_gate(float zr, float zi, float u, float decay, float& la, float& add) {
  const float r = 1.0f / (1.0f + expf(-zr)), i = 1.0f / (1.0f + expf(-zi));
  la = decay * r;
  add = sqrtf(-expm1f(2.0f * la)) * i * u;
}

// The same for the chunks' kernels, whose storage is bfloat16: the hardware's exponential (exp2 of the argument times
// log2 e: a relative error of a few 1e-7) and reciprocal, and 1 - exp(x) for x in -1/2 .. 0 from its Taylor series to the
// ninth power (the next term is less than 1e-9 of the sum), where 1 - exp(x) itself would lose what is left.
__device__ __forceinline__ float one_minus_exp(float x) {
  float p = fmaf(x, 1.0f / 362880, 1.0f / 40320);
  p = fmaf(p, x, 1.0f / 5040);
  p = fmaf(p, x, 1.0f / 720);
  p = fmaf(p, x, 1.0f / 120);
  p = fmaf(p, x, 1.0f / 24);
  p = fmaf(p, x, 1.0f / 6);
  p = fmaf(p, x, 0.5f);
  p = fmaf(p, x, 1.0f);
  return x > -0.5f ? -x * p : 1.0f - __expf(x);
}
__device__ __forceinline__ void lru_gate_fast(float zr, float zi, float u, float decay, float& la, float& add) {
  la = decay * __builtin_amdgcn_rcpf(1.0f + __expf(-zr));
  add = __builtin_amdgcn_sqrtf(one_minus_exp(2.0f * la)) * __builtin_amdgcn_rcpf(1.0f + __expf(-zi)) * u;
}

// V neighbouring outputs of both matrices, summed over one of LRU_SLICES slices of the inner index, two chains an output.
template <typename T, int V>
__device__ __forceinline__ void lru_slice_sums(const float* xs, const T* __restrict__ wr, const T* __restrict__ wi, int n, int c,
                                               int slice, float* sr, float* si) {
  const int per = (n + LRU_SLICES - 1) / LRU_SLICES, i0 = min(n, slice * per), i1 = min(n, i0 + per);
  float r1[V], q1[V];
#pragma unroll
  for (int v = 0; v < V; v++) sr[v] = si[v] = r1[v] = q1[v] = 0.f;
  auto row = [&](const T* w, int i, float* o) {
    const T* p = w + (size_t)i * n + c;
    if constexpr (V == 1) {
      o[0] = load_f32(p);
    } else if constexpr (sizeof(T) == 4) {
      const float2 f = *reinterpret_cast<const float2*>(p);
      o[0] = f.x; o[1] = f.y;
    } else {
      const uint32_t f = *reinterpret_cast<const uint32_t*>(p);
      o[0] = __uint_as_float(f << 16); o[1] = __uint_as_float(f & 0xffff0000u);
    }
  };
  int i = i0;
#pragma unroll 4
  for (; i + 1 < i1; i += 2) {
    float a[V], b[V], c2[V], d[V];
    row(wr, i, a); row(wi, i, b); row(wr, i + 1, c2); row(wi, i + 1, d);
#pragma unroll
    for (int v = 0; v < V; v++) {
      sr[v] = fmaf(xs[i], a[v], sr[v]);
      si[v] = fmaf(xs[i], b[v], si[v]);
      r1[v] = fmaf(xs[i + 1], c2[v], r1[v]);
      q1[v] = fmaf(xs[i + 1], d[v], q1[v]);
    }
  }
  if (i < i1) {
    float a[V], b[V];
    row(wr, i, a); row(wi, i, b);
#pragma unroll
    for (int v = 0; v < V; v++) { sr[v] = fmaf(xs[i], a[v], sr[v]); si[v] = fmaf(xs[i], b[v], si[v]); }
  }
#pragma unroll
  for (int v = 0; v < V; v++) { sr[v] += r1[v]; si[v] += q1[v]; }
}

// The same with the rows in registers, two bfloat16 outputs a word, for slices of at most LRU_AHEAD rows: asked for before
// what they are multiplied with is there.
#define LRU_AHEAD 16
struct LruAhead {
  uint32_t r[LRU_AHEAD], i[LRU_AHEAD];
  __device__ __forceinline__ void load(const bf16_t* __restrict__ wr, const bf16_t* __restrict__ wi, int n, int c, int slice) {
    const int i0 = slice * ((n + LRU_SLICES - 1) / LRU_SLICES);
#pragma unroll
    for (int k = 0; k < LRU_AHEAD; k++) {
      const size_t at = (size_t)min(i0 + k, n - 1) * n + c;
      r[k] = *reinterpret_cast<const uint32_t*>(wr + at);
      i[k] = *reinterpret_cast<const uint32_t*>(wi + at);
    }
  }
  __device__ __forceinline__ void sums(const float* xs, int n, int slice, float* sr, float* si) const {
    const int per = (n + LRU_SLICES - 1) / LRU_SLICES, i0 = min(n, slice * per), i1 = min(n, i0 + per);
    float r1[2] = {0.f, 0.f}, q1[2] = {0.f, 0.f};
    sr[0] = sr[1] = si[0] = si[1] = 0.f;
#pragma unroll
    for (int k = 0; k < LRU_AHEAD; k++) {
      if (i0 + k < i1) {                                  // even rows to one chain, odd rows to the other, as above
        const float x = xs[i0 + k];
        float *a = k & 1 ? r1 : sr, *b = k & 1 ? q1 : si;
        a[0] = fmaf(x, __uint_as_float(r[k] << 16), a[0]);
        a[1] = fmaf(x, __uint_as_float(r[k] & 0xffff0000u), a[1]);
        b[0] = fmaf(x, __uint_as_float(i[k] << 16), b[0]);
        b[1] = fmaf(x, __uint_as_float(i[k] & 0xffff0000u), b[1]);
      }
    }
    sr[0] += r1[0]; sr[1] += r1[1]; si[0] += q1[0]; si[1] += q1[1];
  }
};

__device__ __forceinline__ float lru_slices(const float* part, int width, int c) {
  float s[LRU_SLICES];
#pragma unroll
  for (int k = 0; k < LRU_SLICES; k++) s[k] = part[k * width + c];
  return ((s[0] + s[1]) + (s[2] + s[3])) + ((s[4] + s[5]) + (s[6] + s[7]));
}

// grid (T, blocks, tiles of LRU_TILE outputs), LRU_TILE x LRU_SLICES threads
template <typename T>
__global__ __launch_bounds__(LRU_TILE* LRU_SLICES) void lru_gates_kernel(const T* __restrict__ u, const T* __restrict__ wr,
                                                                         const T* __restrict__ wi, const float* __restrict__ br,
                                                                         const float* __restrict__ bi, const float* __restrict__ decay,
                                                                         float* __restrict__ la, float* __restrict__ add, int C, int n) {
  extern __shared__ float xs[];                           // [n], then [2][slices][tile]
  const int t = blockIdx.x, b = blockIdx.y;
  const T* ur = u + (size_t)t * C + (size_t)b * n;
  for (int i = threadIdx.x; i < n; i += blockDim.x) xs[i] = load_f32(ur + i);
  __syncthreads();
  float* part = xs + n;
  const int cx = threadIdx.x % LRU_TILE, slice = threadIdx.x / LRU_TILE;
  const int c = blockIdx.z * LRU_TILE + cx;
  float sr, si;
  lru_slice_sums<T, 1>(xs, wr + (size_t)b * n * n, wi + (size_t)b * n * n, n, min(c, n - 1), slice, &sr, &si);
  part[slice * LRU_TILE + cx] = sr;
  part[(LRU_SLICES + slice) * LRU_TILE + cx] = si;
  __syncthreads();
  if (slice == 0 && c < n) {
    const int ch = b * n + c;
    const float zr = lru_slices(part, LRU_TILE, cx) + br[ch], zi = lru_slices(part + LRU_SLICES * LRU_TILE, LRU_TILE, cx) + bi[ch];
    float l, a;
    lru_gate(zr, zi, xs[c], decay[ch], l, a);
    la[(size_t)t * C + ch] = l;
    add[(size_t)t * C + ch] = a;
  }
}

// grid (sequences, ceil(C / 64)), 64 threads
template <typename T>
__global__ __launch_bounds__(64) void lru_scan_kernel(const float* __restrict__ la, const float* __restrict__ add,
                                                      const T* __restrict__ y, int ldy, const int* __restrict__ cu_seqlens,
                                                      const int* __restrict__ state_slots, float* __restrict__ state, int num_slots,
                                                      int C, int hist, T* __restrict__ out) {
  const int b = blockIdx.x, c = blockIdx.y * 64 + threadIdx.x;
  const int t_begin = cu_seqlens[b], t_end = cu_seqlens[b + 1], slot = state_slots[b];
  if (c >= C || slot < 0 || slot >= num_slots || t_end <= t_begin) return;
  float* sp = state + ((size_t)slot * C + c) * (1 + hist);
  float S = *sp;
  for (int t0 = t_begin; t0 < t_end; t0 += LRU_TB) {
    const int nb = min(LRU_TB, t_end - t0);
    float l[LRU_TB], a[LRU_TB], yv[LRU_TB];
#pragma unroll
    for (int k = 0; k < LRU_TB; k++) {
      const size_t t = (size_t)(t0 + min(k, nb - 1));
      l[k] = la[t * C + c];
      a[k] = add[t * C + c];
      yv[k] = load_f32(y + t * ldy + c);
    }
#pragma unroll
    for (int k = 0; k < LRU_TB; k++) {
      if (k >= nb) break;
      S = fmaf(expf(l[k]), S, a[k]);
      store_f32(out + (size_t)(t0 + k) * C + c, S * gelu_tanh_f(yv[k]));
    }
  }
  *sp = S;
}

// One token a sequence.  grid (sequences, blocks): a workgroup owns one part of one sequence, so nobody else reads or
// writes the history and the state it brings up to date.  x, y: the convolution's inputs and the gate branch in front of
// its activation, columns of one row each.  TW threads a slice of the inner index, V outputs a thread.  AHEAD: parts whose
// matrices fit the registers of one tile's threads (bfloat16, V 2, n <= LRU_AHEAD x LRU_SLICES, one tile).
template <typename T, int V, bool AHEAD>
__global__ __launch_bounds__(AHEAD ? 512 : 1024) void lru_step_kernel(const T* __restrict__ x, int ldx, const T* __restrict__ y, int ldy,
                                                        const float* __restrict__ conv_w, const float* __restrict__ conv_b,
                                                        const T* __restrict__ wr, const T* __restrict__ wi,
                                                        const float* __restrict__ br, const float* __restrict__ bi,
                                                        const float* __restrict__ decay, const int* __restrict__ cu_seqlens,
                                                        const int* __restrict__ state_slots, float* __restrict__ state, int num_slots,
                                                        int C, int n, int taps, T* __restrict__ out) {
  extern __shared__ float xs[];                           // [n], then [2][slices][V TW]
  const int b = blockIdx.x, blk = blockIdx.y, hist = taps - 1;
  const int t = cu_seqlens[b], slot = state_slots[b];
  if (cu_seqlens[b + 1] != t + 1 || slot < 0 || slot >= num_slots) return;      // the whole workgroup alike
  const int TW = blockDim.x / LRU_SLICES, width = TW * V;
  const int px = threadIdx.x % TW, slice = threadIdx.x / TW;
  const T *wrb = wr + (size_t)blk * n * n, *wib = wi + (size_t)blk * n * n;
  [[maybe_unused]] LruAhead ahead;
  if constexpr (AHEAD) ahead.load(wrb, wib, n, min(px * V, n - V), slice);
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    const int c = blk * n + i;
    float* h = state + ((size_t)slot * C + c) * (1 + hist) + 1;
    const float xv = load_f32(x + (size_t)t * ldx + c);
    float acc = conv_b[c];
    if (hist <= 3) {                                      // the usual few taps: all of them asked for at once
      float v[3], w[4];
#pragma unroll
      for (int j = 0; j < 4; j++) w[j] = conv_w[(size_t)min(j, hist) * C + c];
#pragma unroll
      for (int j = 0; j < 3; j++) v[j] = h[min(j, hist - 1)];       // (no history: the state element in front of it, unused)
#pragma unroll
      for (int j = 0; j < 3; j++)
        if (j < hist) acc = fmaf(w[j], v[j], acc);
      acc = fmaf(hist == 0 ? w[0] : hist == 1 ? w[1] : hist == 2 ? w[2] : w[3], xv, acc);
      if (hist > 0) h[hist - 1] = xv;
      if (hist > 1) h[hist - 2] = hist == 2 ? v[1] : v[2];
      if (hist > 2) h[0] = v[1];
    } else {
      for (int j = 0; j < hist; j++) {
        const float v = h[j];
        acc = fmaf(conv_w[(size_t)j * C + c], v, acc);
        if (j > 0) h[j - 1] = v;
      }
      acc = fmaf(conv_w[(size_t)hist * C + c], xv, acc);
      h[hist - 1] = xv;
    }
    T u;
    store_f32(&u, acc);                                   // as the convolution's own launch leaves it, in the storage type
    xs[i] = load_f32(&u);
  }
  __syncthreads();
  float* part = xs + n;
  for (int c0 = 0; c0 < n; c0 += width) {
    // what the last part of the loop needs travels under the products
    const int ce = c0 + (int)threadIdx.x, ch = blk * n + min(ce, n - 1);
    const bool mine = (int)threadIdx.x < width && ce < n;
    float* sp = state + ((size_t)slot * C + ch) * (1 + hist);
    float S = 0.f, yv = 0.f, dec = 0.f, b_r = 0.f, b_i = 0.f;
    if (mine) { S = *sp; yv = load_f32(y + (size_t)t * ldy + ch); dec = decay[ch]; b_r = br[ch]; b_i = bi[ch]; }
    const int c = c0 + px * V;
    float sr[V], si[V];
    if constexpr (AHEAD) ahead.sums(xs, n, slice, sr, si);
    else lru_slice_sums<T, V>(xs, wrb, wib, n, min(c, n - V), slice, sr, si);
    __syncthreads();                                      // the last tile's sums have been read
#pragma unroll
    for (int v = 0; v < V; v++) {
      part[slice * width + px * V + v] = sr[v];
      part[(LRU_SLICES + slice) * width + px * V + v] = si[v];
    }
    __syncthreads();
    if (mine) {
      const float zr = lru_slices(part, width, threadIdx.x) + b_r, zi = lru_slices(part + LRU_SLICES * width, width, threadIdx.x) + b_i;
      float l, a;
      lru_gate(zr, zi, xs[ce], dec, l, a);
      S = fmaf(expf(l), S, a);
      *sp = S;
      store_f32(out + (size_t)t * C + ch, S * gelu_tanh_f(yv));
    }
  }
}

// grid (sequences * max_chunks, blocks, ceil(n / 64)), four waves.  Wave w makes both gates of tokens 16 w .. 16 w + 15 for 64
// outputs (16x16x32 products: lane (i, g) holds row i, inner indices 8 g .. 8 g + 7 of both operands, and of a result column
// i, rows 4 g + 0..3), then walks its 16 tokens with a lane a channel.
__global__ __launch_bounds__(256) void lru_gates_chunk_kernel(const bf16_t* __restrict__ u, const bf16_t* __restrict__ wr,
                                                              const bf16_t* __restrict__ wi, const float* __restrict__ br,
                                                              const float* __restrict__ bi, const float* __restrict__ decay,
                                                              const int* __restrict__ cu_seqlens, int C, int n, int max_chunks,
                                                              float* __restrict__ local, float* __restrict__ sum_la,
                                                              float* __restrict__ ws_s, float* __restrict__ ws_la) {
  constexpr int LD = 68;                                   // floats a token: the four row groups of a store land on other banks
  __shared__ float la[LRU_CHUNK][LD], add[LRU_CHUNK][LD];
  __shared__ float end_s[4][64], end_la[4][64];
  const int seq = blockIdx.x / max_chunks, blk = blockIdx.y, out0 = blockIdx.z * 64;
  const int t_begin = cu_seqlens[seq] + (blockIdx.x % max_chunks) * LRU_CHUNK;
  const int t_end = min(cu_seqlens[seq + 1], t_begin + LRU_CHUNK);
  if (t_end <= t_begin) return;                            // the whole workgroup alike
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4;
  const bf16_t* ub = u + (size_t)blk * n;
  const bf16_t* arow = ub + (size_t)min(t_begin + 16 * wave + i, t_end - 1) * C;
  const bf16_t *rrow[4], *irow[4];
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const size_t o = ((size_t)blk * n + min(out0 + 16 * j + i, n - 1)) * n;
    rrow[j] = wr + o;
    irow[j] = wi + o;
  }
  f32x4 zr[4], zi[4];
#pragma unroll
  for (int j = 0; j < 4; j++) zr[j] = zi[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const u32x4 none = {0u, 0u, 0u, 0u};
  // what the gates read beside their products travels under them
  float b_r[4], b_i[4], dec[4];
  bf16_t uv[4][4];
#pragma unroll
  for (int j = 0; j < 4; j++) {
    const int c = min(out0 + 16 * j + i, n - 1), ch = blk * n + c;
    b_r[j] = br[ch]; b_i[j] = bi[ch]; dec[j] = decay[ch];
#pragma unroll
    for (int q = 0; q < 4; q++) uv[j][q] = ub[(size_t)min(t_begin + 16 * wave + 4 * g + q, t_end - 1) * C + c];
  }
  for (int k0 = 0; k0 < n; k0 += 64) {                     // two products' operands at a time
    u32x4 a[2], r4[2][4], i4[2][4];
#pragma unroll
    for (int h = 0; h < 2; h++) {
      const int ks = min(k0 + 32 * h + 8 * g, n - 8);      // n is a multiple of 8; behind its end both operands read as zero
      a[h] = *reinterpret_cast<const u32x4*>(arow + ks);
#pragma unroll
      for (int j = 0; j < 4; j++) {
        r4[h][j] = *reinterpret_cast<const u32x4*>(rrow[j] + ks);
        i4[h][j] = *reinterpret_cast<const u32x4*>(irow[j] + ks);
      }
    }
#pragma unroll
    for (int h = 0; h < 2; h++) {
      const bool in = k0 + 32 * h + 8 * g < n;
      a[h] = in ? a[h] : none;
#pragma unroll
      for (int j = 0; j < 4; j++) {
        r4[h][j] = in ? r4[h][j] : none;
        i4[h][j] = in ? i4[h][j] : none;
        zr[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a[h]), __builtin_bit_cast(bf16x8, r4[h][j]), zr[j], 0, 0, 0);
        zi[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a[h]), __builtin_bit_cast(bf16x8, i4[h][j]), zi[j], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < 4; j++) {
#pragma unroll
    for (int q = 0; q < 4; q++) {
      const int k = 16 * wave + 4 * g + q;
      float l, ad;
      lru_gate_fast(zr[j][q] + b_r[j], zi[j][q] + b_i[j], bf16_to_f32(uv[j][q]), dec[j], l, ad);
      if (t_begin + k >= t_end) l = ad = 0.f;              // a token behind the chunk's end changes nothing
      la[k][16 * j + i] = l;
      add[k][16 * j + i] = ad;
    }
  }
  __syncthreads();
  float s[16], L[16];
#pragma unroll
  for (int k = 0; k < 16; k++) {
    L[k] = la[16 * wave + k][lane];
    s[k] = add[16 * wave + k][lane];
  }
#pragma unroll
  for (int k = 1; k < 16; k++) {
    s[k] = fmaf(__expf(L[k]), s[k - 1], s[k]);
    L[k] += L[k - 1];
  }
  end_s[wave][lane] = s[15];
  end_la[wave][lane] = L[15];
  __syncthreads();
  float S0 = 0.f, L0 = 0.f;
  for (int v = 0; v < wave; v++) {
    S0 = fmaf(__expf(end_la[v][lane]), S0, end_s[v][lane]);
    L0 += end_la[v][lane];
  }
  const int c = out0 + lane;
  if (c >= n) return;
  const size_t ch = (size_t)blk * n + c;
#pragma unroll
  for (int k = 0; k < 16; k++) {
    const int t = t_begin + 16 * wave + k;
    if (t < t_end) {
      local[(size_t)t * C + ch] = fmaf(__expf(L[k]), S0, s[k]);
      sum_la[(size_t)t * C + ch] = L0 + L[k];
    }
  }
  if (wave == 3) {
    ws_s[(size_t)blockIdx.x * C + ch] = fmaf(__expf(L[15]), S0, s[15]);
    ws_la[(size_t)blockIdx.x * C + ch] = L0 + L[15];
  }
}

// grid (sequences, ceil(C / 64)), 64 threads: ws_s[j] becomes the state in front of chunk j, the slot gets the last state.
__global__ __launch_bounds__(64) void lru_combine_kernel(const int* __restrict__ cu_seqlens, const int* __restrict__ state_slots,
                                                         float* __restrict__ state, float* __restrict__ ws_s,
                                                         const float* __restrict__ ws_la, int num_slots, int C, int hist,
                                                         int max_chunks) {
  const int b = blockIdx.x, c = blockIdx.y * 64 + threadIdx.x;
  const int n_tok = cu_seqlens[b + 1] - cu_seqlens[b], slot = state_slots[b];
  if (c >= C || slot < 0 || slot >= num_slots || n_tok <= 0) return;
  float* sp = state + ((size_t)slot * C + c) * (1 + hist);
  float S = *sp;
  const int chunks = (n_tok + LRU_CHUNK - 1) / LRU_CHUNK;
  for (int j0 = 0; j0 < chunks; j0 += LRU_TB) {
    float s[LRU_TB], l[LRU_TB];
#pragma unroll
    for (int k = 0; k < LRU_TB; k++) {                     // sixteen chunks' values travel together
      const size_t at = ((size_t)b * max_chunks + min(j0 + k, chunks - 1)) * C + c;
      s[k] = ws_s[at];
      l[k] = ws_la[at];
    }
#pragma unroll
    for (int k = 0; k < LRU_TB; k++) {
      if (j0 + k >= chunks) break;
      ws_s[((size_t)b * max_chunks + j0 + k) * C + c] = S;
      S = fmaf(expf(l[k]), S, s[k]);
    }
  }
  *sp = S;
}

// grid (T, ceil(C / 4 / 256)): four neighbouring channels a thread (C a multiple of 8)
__global__ __launch_bounds__(256) void lru_chunk_out_kernel(const float* __restrict__ local, const float* __restrict__ sum_la,
                                                            const float* __restrict__ ws_s, const bf16_t* __restrict__ y, int ldy,
                                                            const int* __restrict__ token_seq, const int* __restrict__ cu_seqlens,
                                                            int C, int max_chunks, bf16_t* __restrict__ out) {
  const int t = blockIdx.x, c = (blockIdx.y * blockDim.x + threadIdx.x) * 4;
  if (c >= C) return;
  const int b = token_seq[t], j = (t - cu_seqlens[b]) / LRU_CHUNK;
  const float4 h = *reinterpret_cast<const float4*>(local + (size_t)t * C + c);
  const float4 l = *reinterpret_cast<const float4*>(sum_la + (size_t)t * C + c);
  const float4 s = *reinterpret_cast<const float4*>(ws_s + ((size_t)b * max_chunks + j) * C + c);
  const bf16_t* yr = y + (size_t)t * ldy + c;
  uint2 o;
  o.x = pack2_bf16(fmaf(__expf(l.x), s.x, h.x) * gelu_tanh_f(bf16_to_f32(yr[0])), fmaf(__expf(l.y), s.y, h.y) * gelu_tanh_f(bf16_to_f32(yr[1])));
  o.y = pack2_bf16(fmaf(__expf(l.z), s.z, h.z) * gelu_tanh_f(bf16_to_f32(yr[2])), fmaf(__expf(l.w), s.w, h.w) * gelu_tanh_f(bf16_to_f32(yr[3])));
  *reinterpret_cast<uint2*>(out + (size_t)t * C + c) = o;
}

#define LRU_CHECK(who)                                                                                                    \
  PICO_REQUIRE(T >= 0 && B >= 0 && C > 0 && blocks > 0 && C % blocks == 0 && C / blocks <= LRU_MAX_N && blocks <= 65535 && \
                   num_slots > 0 && hist >= 0 && hist < LRU_MAX_TAPS && ldy >= C && (dtype | 1) == 1,                     \
               who ": bad sizes (parts of at most %d channels, at most %d taps)", LRU_MAX_N, LRU_MAX_TAPS)

// Gates and walk: u [T, C]; wr, wi [blocks, inner, output]; la, add: float32 [T, C], room for what the gates leave.
extern "C" int pico_lru_scan(const void* u, const void* y, int ldy, int dtype, const void* wr, const void* wi, const float* br,
                             const float* bi, const float* decay, const int* cu_seqlens, const int* state_slots, float* state,
                             int num_slots, int T, int B, int C, int blocks, int hist, float* la, float* add, void* out,
                             hipStream_t stream) {
  LRU_CHECK("pico_lru_scan");
  if (T == 0 || B == 0) return 0;
  const int n = C / blocks;
  const dim3 grid(T, blocks, (n + LRU_TILE - 1) / LRU_TILE), sgrid(B, (C + 63) / 64);
  const size_t lds = (size_t)(n + 2 * LRU_SLICES * LRU_TILE) * sizeof(float);
  if (dtype == PICO_DTYPE_F32) {
    lru_gates_kernel<float><<<grid, LRU_TILE * LRU_SLICES, lds, stream>>>((const float*)u, (const float*)wr, (const float*)wi, br, bi, decay, la, add, C, n);
    lru_scan_kernel<float><<<sgrid, 64, 0, stream>>>(la, add, (const float*)y, ldy, cu_seqlens, state_slots, state, num_slots, C, hist, (float*)out);
  } else {
    lru_gates_kernel<bf16_t><<<grid, LRU_TILE * LRU_SLICES, lds, stream>>>((const bf16_t*)u, (const bf16_t*)wr, (const bf16_t*)wi, br, bi, decay, la, add, C, n);
    lru_scan_kernel<bf16_t><<<sgrid, 64, 0, stream>>>(la, add, (const bf16_t*)y, ldy, cu_seqlens, state_slots, state, num_slots, C, hist, (bf16_t*)out);
  }
  PICO_LAUNCH_CHECK();
  return 0;
}

// One token a sequence (T == B): x [T, C] the convolution's inputs (rows ldx apart), conv_w [taps, C] tap by tap.
extern "C" int pico_lru_step(const void* x, int ldx, const void* y, int ldy, int dtype, const float* conv_w, const float* conv_b,
                             const void* wr, const void* wi, const float* br, const float* bi, const float* decay,
                             const int* cu_seqlens, const int* state_slots, float* state, int num_slots, int T, int B, int C,
                             int blocks, int hist, void* out, hipStream_t stream) {
  LRU_CHECK("pico_lru_step");
  PICO_REQUIRE(T == B && ldx >= C, "pico_lru_step: one token a sequence, and rows that hold the channels");
  if (B == 0) return 0;
  const int n = C / blocks, taps = hist + 1;
  const bool two = n % 2 == 0;
  const int units = two ? n / 2 : n;
  const int tw = min(128, (units + 7) / 8 * 8);
  const size_t lds = (size_t)(n + 2 * LRU_SLICES * tw * (two ? 2 : 1)) * sizeof(float);
  const dim3 grid(B, blocks);
#define LAUNCH(TT, V, AHEAD)                                                                                                       \
  lru_step_kernel<TT, V, AHEAD><<<grid, tw * LRU_SLICES, lds, stream>>>((const TT*)x, ldx, (const TT*)y, ldy, conv_w, conv_b, (const TT*)wr, \
                                                                 (const TT*)wi, br, bi, decay, cu_seqlens, state_slots, state,     \
                                                                 num_slots, C, n, taps, (TT*)out)
  if (dtype == PICO_DTYPE_F32) {
    if (two) LAUNCH(float, 2, false); else LAUNCH(float, 1, false);
  } else {
    if (two && n <= LRU_AHEAD * LRU_SLICES) LAUNCH(bf16_t, 2, true);       // (one tile of at most 512 threads)
    else if (two) LAUNCH(bf16_t, 2, false);
    else LAUNCH(bf16_t, 1, false);
  }
#undef LAUNCH
  PICO_LAUNCH_CHECK();
  return 0;
}

// Chunks side by side, bfloat16: wr, wi [blocks, output, inner]; local, sum_la float32 [T, C]; ws_s, ws_la float32
// [B * max_chunks, C]; max_chunks at least the chunks of the longest sequence.
extern "C" int pico_lru_chunks(const void* u, const void* y, int ldy, int dtype, const void* wr, const void* wi, const float* br,
                               const float* bi, const float* decay, const int* token_seq, const int* cu_seqlens,
                               const int* state_slots, float* state, int num_slots, int T, int B, int C, int blocks, int hist,
                               int max_chunks, float* local, float* sum_la, float* ws_s, float* ws_la, void* out, hipStream_t stream) {
  LRU_CHECK("pico_lru_chunks");
  PICO_REQUIRE(dtype == PICO_DTYPE_BF16 && (C / blocks) % 8 == 0, "pico_lru_chunks: bfloat16, parts of a multiple of 8 channels");
  PICO_REQUIRE((uintptr_t)u % 16 == 0 && (uintptr_t)wr % 16 == 0 && (uintptr_t)wi % 16 == 0 && (uintptr_t)out % 16 == 0 &&
                   (uintptr_t)local % 16 == 0 && (uintptr_t)sum_la % 16 == 0 && (uintptr_t)ws_s % 16 == 0,
               "pico_lru_chunks: operands must be 16-byte aligned");
  PICO_REQUIRE(max_chunks > 0 && (long long)max_chunks * LRU_CHUNK >= T && (long long)B * max_chunks < (1ll << 31),
               "pico_lru_chunks: the chunks must cover the step's tokens");
  if (T == 0 || B == 0) return 0;
  const int n = C / blocks;
  lru_gates_chunk_kernel<<<dim3(B * max_chunks, blocks, (n + 63) / 64), 256, 0, stream>>>(
      (const bf16_t*)u, (const bf16_t*)wr, (const bf16_t*)wi, br, bi, decay, cu_seqlens, C, n, max_chunks, local, sum_la, ws_s, ws_la);
  lru_combine_kernel<<<dim3(B, (C + 63) / 64), 64, 0, stream>>>(cu_seqlens, state_slots, state, ws_s, ws_la, num_slots, C, hist, max_chunks);
  lru_chunk_out_kernel<<<dim3(T, (C / 4 + 255) / 256), 256, 0, stream>>>(local, sum_la, ws_s, (const bf16_t*)y, ldy, token_seq, cu_seqlens,
                                                                         C, max_chunks, (bf16_t*)out);
  PICO_LAUNCH_CHECK();
  return 0;
}
