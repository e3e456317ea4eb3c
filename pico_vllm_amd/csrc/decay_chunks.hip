// Linear attention with a constant decay a head (the recurrence of gla.hip with one number in place of a token's decays), in
// chunks that run side by side on the matrix cores:
//
//   S_t = g S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t          (per head; g the head's decay, S [dk, dv])
//
// With i, j counted inside a chunk of n <= 64 tokens and S0 the state in front of it
//
//   o_i = sum_(j <= i) g^(i - j) (q_i . k_j) v_j + g^(i + 1) S0^T q_i
//   S_n = g^n S0 + L,   L = sum_j g^(n - 1 - j) k_j v_j^T
//
// Three launches: every chunk's L from zero; a walk over a sequence's chunks that turns the L's into the states in front
// of the chunks and leaves the slot's new state; every chunk's outputs.  The operands are bfloat16 rows (optionally through
// z sigmoid(z) as they are read); from there on everything is float32, the products included (v_mfma_f32_32x32x2_f32), so
// state, decays and sums are what the walk's are, in another order.
//
// A workgroup (four waves) owns one chunk, one head and 32 NBLK value columns; its rows lie in LDS as float32.  An operand
// tile of the products is 32 rows (lane % 32) by 2 k (lane / 32); which k a step takes is free as long as both operands
// agree, so lane half h takes k = 8 b + 4 h + 0..3 over four steps: four contiguous floats where k runs along a row.
#include "common.h"

typedef float f32x16 __attribute__((ext_vector_type(16)));

#define DC_CHUNK 64

struct ChunkArgs {
  const bf16_t* x;             // [T, ld]; q, k, v of head h from columns q_col + h dk, k_col + h dk, v_col + h dv
  int ld, q_col, k_col, v_col;
  const int* cu_seqlens;
  const int* state_slots;
  const float* decay;          // [H]
  float* state;                // [slots, H, dk, dv]
  float* ws;                   // [sequences * max_chunks, H, dk, dv]
  float* out;                  // [T, H dv]
  int H, dk, dv, num_slots, max_chunks, silu;
  float qscale;
};

// g^n for n >= 0 (lg = log2 g); g = 1 exactly stays 1
__device__ __forceinline__ float decay_power(float lg, int n) { return exp2f(lg * (float)n); }

__device__ __forceinline__ float act8(uint32_t w, bool high, int silu) {
  const float z = high ? __uint_as_float(w & 0xffff0000u) : __uint_as_float(w << 16);
  return silu ? z / (1.0f + __expf(-z)) : z;
}

// A thread's pieces (8 columns of a row each) of 64 rows x COLS columns: asked for by `fetch`, written to LDS by `put`.
// Rows from n on and columns from `cols` on (a multiple of 8) read as zero; every load is from an address inside.
template <int COLS>
struct Rows {
  static constexpr int N = DC_CHUNK * COLS / 8 / 256;
  static_assert(N >= 1, "at least one piece a thread");
  uint4 v[N];
  __device__ __forceinline__ void fetch(const bf16_t* src, int ld, int n, int cols) {
#pragma unroll
    for (int i = 0; i < N; i++) {
      const int u = threadIdx.x + 256 * i, r = u / (COLS / 8), c = u % (COLS / 8) * 8;
      v[i] = *reinterpret_cast<const uint4*>(src + (size_t)min(r, n - 1) * ld + (c < cols ? c : 0));
    }
  }
  template <typename F>
  __device__ __forceinline__ void put(float* dst, int stride, int n, int cols, int silu, F factor) {
#pragma unroll
    for (int i = 0; i < N; i++) {
      const int u = threadIdx.x + 256 * i, r = u / (COLS / 8), c = u % (COLS / 8) * 8;
      const float f = (r < n && c < cols) ? factor(r) : 0.f;
      float4 a, b;
      a.x = act8(v[i].x, false, silu) * f; a.y = act8(v[i].x, true, silu) * f;
      a.z = act8(v[i].y, false, silu) * f; a.w = act8(v[i].y, true, silu) * f;
      b.x = act8(v[i].z, false, silu) * f; b.y = act8(v[i].z, true, silu) * f;
      b.z = act8(v[i].w, false, silu) * f; b.w = act8(v[i].w, true, silu) * f;
      if (!(r < n && c < cols)) a = b = make_float4(0.f, 0.f, 0.f, 0.f);
      *reinterpret_cast<float4*>(dst + r * stride + c) = a;
      *reinterpret_cast<float4*>(dst + r * stride + c + 4) = b;
    }
  }
};

__device__ __forceinline__ f32x16 mfma32(float a, float b, f32x16 c) { return __builtin_amdgcn_mfma_f32_32x32x2f32(a, b, c, 0, 0, 0); }

__device__ __forceinline__ f32x16 zero16() {
  f32x16 z;
#pragma unroll
  for (int r = 0; r < 16; r++) z[r] = 0.f;
  return z;
}

// which tokens a workgroup has; false: none
__device__ __forceinline__ bool chunk_tokens(const ChunkArgs& a, int& t0, int& n) {
  const int b = blockIdx.x / a.max_chunks;
  t0 = a.cu_seqlens[b] + blockIdx.x % a.max_chunks * DC_CHUNK;
  n = min(DC_CHUNK, a.cu_seqlens[b + 1] - t0);
  const int slot = a.state_slots[b];
  return n > 0 && slot >= 0 && slot < a.num_slots;
}

// L of every chunk into ws.  Wave w: value columns 32 (w % NBLK) .. of the workgroup's; with fewer than four column blocks
// the waves of one share the key channels.
template <int DKP, int NBLK>
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(const ChunkArgs a) {
  constexpr int KS = DKP + 4, NB = 32 * NBLK, VS = NB + 8, CB = DKP / 32, SHARE = 4 / NBLK;
  __shared__ __attribute__((aligned(16))) float ks[DC_CHUNK * KS];
  __shared__ __attribute__((aligned(16))) float vs[DC_CHUNK * VS];
  int t0, n;
  if (!chunk_tokens(a, t0, n)) return;
  const int h = blockIdx.y, n0 = blockIdx.z * NB, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l = lane & 31, half = lane >> 5;
  const float lg = log2f(a.decay[h]);
  const bf16_t* row = a.x + (size_t)t0 * a.ld;
  Rows<DKP> k;
  Rows<NB> v;
  k.fetch(row + a.k_col + h * a.dk, a.ld, n, a.dk);
  v.fetch(row + a.v_col + h * a.dv + n0, a.ld, n, a.dv - n0);
  k.put(ks, KS, n, a.dk, a.silu, [&](int r) { return decay_power(lg, n - 1 - r); });
  v.put(vs, VS, n, a.dv - n0, a.silu, [&](int) { return 1.0f; });
  __syncthreads();
  const int nb = wave % NBLK, c_first = wave / NBLK;
  const float* vp = vs + 4 * half * VS + 32 * nb + l;
  f32x16 acc[(CB + SHARE - 1) / SHARE];
#pragma unroll
  for (int i = 0; i < (CB + SHARE - 1) / SHARE; i++) acc[i] = zero16();
#pragma unroll 2
  for (int j = 0; j < DC_CHUNK; j += 8) {
    float b[4];
#pragma unroll
    for (int s = 0; s < 4; s++) b[s] = vp[(j + s) * VS];
#pragma unroll
    for (int i = 0; i < (CB + SHARE - 1) / SHARE; i++) {
      const int cb = min(c_first + i * SHARE, CB - 1);
      const float* kp = ks + (j + 4 * half) * KS + 32 * cb + l;
#pragma unroll
      for (int s = 0; s < 4; s++) acc[i] = mfma32(kp[s * KS], b[s], acc[i]);
    }
  }
  float* ws = a.ws + ((size_t)blockIdx.x * a.H + h) * a.dk * a.dv;
  const int col = n0 + 32 * nb + l;
  if (col >= a.dv) return;
#pragma unroll
  for (int i = 0; i < (CB + SHARE - 1) / SHARE; i++) {
    const int cb = c_first + i * SHARE;
    if (cb >= CB) break;
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int c = 32 * cb + 8 * (r >> 2) + 4 * half + (r & 3);
      if (c < a.dk) ws[(size_t)c * a.dv + col] = acc[i][r];
    }
  }
}

// The walk over a sequence's chunks, a thread a state element: ws becomes the state in front of every chunk, the slot gets
// the state behind the last.  The loads of DC_AHEAD chunks travel together.  grid (sequences, heads, ceil(dk dv / 256)).
#define DC_AHEAD 8
__global__ __launch_bounds__(256) void decay_chunk_walk_kernel(const ChunkArgs a) {
  const int b = blockIdx.x, h = blockIdx.y, size = a.dk * a.dv, e = blockIdx.z * 256 + threadIdx.x;
  if (e >= size) return;
  const int slot = a.state_slots[b], n = a.cu_seqlens[b + 1] - a.cu_seqlens[b];
  if (slot < 0 || slot >= a.num_slots || n <= 0) return;
  const float lg = log2f(a.decay[h]), whole = decay_power(lg, DC_CHUNK);
  float* sp = a.state + ((size_t)slot * a.H + h) * size + e;
  float* w = a.ws + ((size_t)b * a.max_chunks * a.H + h) * size + e;
  const size_t step = (size_t)a.H * size;
  const int chunks = (n + DC_CHUNK - 1) / DC_CHUNK;
  float S = *sp;
  for (int j0 = 0; j0 < chunks; j0 += DC_AHEAD) {
    float local[DC_AHEAD];
#pragma unroll
    for (int i = 0; i < DC_AHEAD; i++) local[i] = w[min(j0 + i, chunks - 1) * step];
#pragma unroll
    for (int i = 0; i < DC_AHEAD; i++) {
      if (j0 + i >= chunks) break;
      w[(j0 + i) * step] = S;
      const int left = n - (j0 + i) * DC_CHUNK;
      S = fmaf(left < DC_CHUNK ? decay_power(lg, left) : whole, S, local[i]);
    }
  }
  *sp = S;
}

// The outputs of every chunk.  Wave w: value columns 32 (w % NBLK) ..; with four column blocks it makes both blocks of 32
// tokens, with two one of them.  Products of queries and keys are made by three waves (the block of later keys and earlier
// queries is empty) and meet the values through LDS, where they take the keys' place.
template <int DKP, int NBLK>
__global__ __launch_bounds__(256) void decay_chunk_out_kernel(const ChunkArgs a) {
  constexpr int KS = DKP + 4, PS = DC_CHUNK + 4, NB = 32 * NBLK, VS = NB + 8, IB = NBLK == 4 ? 2 : 1;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* qs = lds;
  float* ks = qs + DC_CHUNK * KS;                        // the keys, then the weighted products [64][PS]
  float* vs = ks + DC_CHUNK * (KS > PS ? KS : PS);
  int t0, n;
  if (!chunk_tokens(a, t0, n)) return;
  const int h = blockIdx.y, n0 = blockIdx.z * NB, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l = lane & 31, half = lane >> 5;
  const int nb = wave % NBLK, ib0 = NBLK == 4 ? 0 : wave / NBLK, col = n0 + 32 * nb + l;
  const float lg = log2f(a.decay[h]);
  const bf16_t* row = a.x + (size_t)t0 * a.ld;
  Rows<DKP> q, k;
  Rows<NB> v;
  q.fetch(row + a.q_col + h * a.dk, a.ld, n, a.dk);
  k.fetch(row + a.k_col + h * a.dk, a.ld, n, a.dk);
  v.fetch(row + a.v_col + h * a.dv + n0, a.ld, n, a.dv - n0);
  // the state in front of the chunk as an operand: rows 8 b + 4 half + 0..3, this lane's column
  float s0[DKP / 2];
  {
    const float* sp = a.ws + ((size_t)blockIdx.x * a.H + h) * a.dk * a.dv + min(col, a.dv - 1);
#pragma unroll
    for (int i = 0; i < DKP / 2; i++) s0[i] = sp[(size_t)min(i / 4 * 8 + 4 * half + i % 4, a.dk - 1) * a.dv];
  }
  q.put(qs, KS, n, a.dk, a.silu, [&](int) { return a.qscale; });
  k.put(ks, KS, n, a.dk, a.silu, [&](int) { return 1.0f; });
  v.put(vs, VS, n, a.dv - n0, a.silu, [&](int) { return 1.0f; });
  __syncthreads();
  // queries and keys: wave 0 block (0, 0), wave 1 (1, 0), wave 2 (1, 1)
  const int pi = wave == 0 ? 0 : 1, pj = wave == 2 ? 1 : 0;
  f32x16 p = zero16();
  if (wave < 3) {
    const float* qp = qs + (32 * pi + l) * KS + 4 * half;
    const float* kp = ks + (32 * pj + l) * KS + 4 * half;
#pragma unroll 4
    for (int c = 0; c < DKP; c += 8) {
      const float4 qv = *reinterpret_cast<const float4*>(qp + c), kv = *reinterpret_cast<const float4*>(kp + c);
      p = mfma32(qv.x, kv.x, p);
      p = mfma32(qv.y, kv.y, p);
      p = mfma32(qv.z, kv.z, p);
      p = mfma32(qv.w, kv.w, p);
    }
  }
  // what the state contributes
  f32x16 acc[IB];
#pragma unroll
  for (int i = 0; i < IB; i++) acc[i] = zero16();
#pragma unroll
  for (int c = 0; c < DKP; c += 8) {
#pragma unroll
    for (int i = 0; i < IB; i++) {
      const float4 qv = *reinterpret_cast<const float4*>(qs + (32 * (ib0 + i) + l) * KS + 4 * half + c);
      // (rows of the state from dk on stand beside zeros of q; they are another row's numbers, finite as the state is)
      acc[i] = mfma32(qv.x, s0[c / 2], acc[i]);
      acc[i] = mfma32(qv.y, s0[c / 2 + 1], acc[i]);
      acc[i] = mfma32(qv.z, s0[c / 2 + 2], acc[i]);
      acc[i] = mfma32(qv.w, s0[c / 2 + 3], acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < IB; i++)
#pragma unroll
    for (int r = 0; r < 16; r++) acc[i][r] *= decay_power(lg, 32 * (ib0 + i) + 8 * (r >> 2) + 4 * half + (r & 3) + 1);
  __syncthreads();                                       // every wave is done with the keys
  if (wave < 3) {
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int i = 32 * pi + 8 * (r >> 2) + 4 * half + (r & 3), j = 32 * pj + l;
      ks[i * PS + j] = j <= i ? p[r] * decay_power(lg, i - j) : 0.f;
    }
  }
  __syncthreads();
  const float* vp = vs + 4 * half * VS + 32 * nb + l;
#pragma unroll
  for (int i = 0; i < IB; i++) {
    const int ib = ib0 + i;
    const float* pp = ks + (32 * ib + l) * PS + 4 * half;
#pragma unroll 4
    for (int j = 0; j < 32 * (ib + 1); j += 8) {
      const float4 pv = *reinterpret_cast<const float4*>(pp + j);
      acc[i] = mfma32(pv.x, vp[j * VS], acc[i]);
      acc[i] = mfma32(pv.y, vp[(j + 1) * VS], acc[i]);
      acc[i] = mfma32(pv.z, vp[(j + 2) * VS], acc[i]);
      acc[i] = mfma32(pv.w, vp[(j + 3) * VS], acc[i]);
    }
  }
  if (col >= a.dv) return;
#pragma unroll
  for (int i = 0; i < IB; i++)
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int t = 32 * (ib0 + i) + 8 * (r >> 2) + 4 * half + (r & 3);
      if (t < n) a.out[(size_t)(t0 + t) * a.H * a.dv + (size_t)h * a.dv + col] = acc[i][r];
    }
}

template <int DKP, int NBLK>
static int launch_chunks(const ChunkArgs& a, int num_seqs, hipStream_t stream) {
  constexpr int KS = DKP + 4, PS = DC_CHUNK + 4, VS = 32 * NBLK + 8;
  constexpr int bytes = DC_CHUNK * (KS + (KS > PS ? KS : PS) + VS) * (int)sizeof(float);
  static bool raised = false;
  if (!raised) {
    PICO_REQUIRE(hipFuncSetAttribute((const void*)decay_chunk_out_kernel<DKP, NBLK>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes) == hipSuccess,
                 "pico_decay_chunks: %d bytes of LDS refused", bytes);
    raised = true;
  }
  const dim3 grid(num_seqs * a.max_chunks, a.H, (a.dv + 32 * NBLK - 1) / (32 * NBLK));
  decay_chunk_state_kernel<DKP, NBLK><<<grid, 256, 0, stream>>>(a);
  decay_chunk_walk_kernel<<<dim3(num_seqs, a.H, (a.dk * a.dv + 255) / 256), 256, 0, stream>>>(a);
  decay_chunk_out_kernel<DKP, NBLK><<<grid, 256, bytes, stream>>>(a);
  PICO_LAUNCH_CHECK();
  return 0;
}

extern "C" int pico_decay_chunk_tokens() { return DC_CHUNK; }

// x bfloat16 [T, ld]; ws float32 [num_seqs * max_chunks, H, dk, dv], max_chunks at least the chunks of the longest sequence.
extern "C" int pico_decay_chunks(const void* x, int ld, int q_col, int k_col, int v_col, const int* cu_seqlens, const int* state_slots,
                                 const float* decay, float* state, float* out, float* ws, int num_seqs, int T, int H, int dk, int dv,
                                 float qscale, int num_slots, int max_chunks, int silu, hipStream_t stream) {
  PICO_REQUIRE(num_seqs >= 0 && T >= 0 && H > 0 && H <= 65535 && dk > 0 && dv > 0 && num_slots > 0, "pico_decay_chunks: bad sizes");
  PICO_REQUIRE(dk <= 128 && dk % 8 == 0 && dv % 8 == 0, "pico_decay_chunks: keys of a multiple of 8 up to 128 and values of a multiple of 8, got %d and %d", dk, dv);
  PICO_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && ld >= q_col + H * dk && ld >= k_col + H * dk && ld >= v_col + H * dv,
               "pico_decay_chunks: the row of %d columns does not hold q, k and v", ld);
  PICO_REQUIRE((ld | q_col | k_col | v_col) % 8 == 0 && (uintptr_t)x % 16 == 0, "pico_decay_chunks: rows and columns must start on 16 bytes");
  PICO_REQUIRE(max_chunks > 0 && (long long)max_chunks * DC_CHUNK >= T && (long long)num_seqs * max_chunks < (1ll << 31) && ws && state && out && decay,
               "pico_decay_chunks: chunks need room for their states and must cover the step's tokens");
  PICO_REQUIRE((dv + 63) / 64 <= 65535 && (dk * dv + 255) / 256 <= 65535, "pico_decay_chunks: sizes beyond the grid");
  if (num_seqs == 0 || T == 0) return 0;
  const ChunkArgs a{(const bf16_t*)x, ld, q_col, k_col, v_col, cu_seqlens, state_slots, decay, state, ws, out, H, dk, dv, num_slots, max_chunks, silu, qscale};
  const bool wide = dv > 64;
#define PICK(DKP) return wide ? launch_chunks<DKP, 4>(a, num_seqs, stream) : launch_chunks<DKP, 2>(a, num_seqs, stream)
  if (dk <= 32) PICK(32);
  if (dk <= 64) PICK(64);
  if (dk <= 96) PICK(96);
  PICK(128);
#undef PICK
}
