// A step of single tokens of two mixers side by side, attention and linear attention with a constant decay a head, between
// their joint products (bfloat16 rows): what the two do beside each other shares a launch, in workgroups of either kind.
//
//   pico_pair_open:   attention: unit norm of the query and key heads, rotation of neighbours, store of keys and values (as
//                     pico_qk_norm_store without weights);  linear attention: S <- g S + k v^T, o = S^T q (as
//                     pico_gla_scan, one token a sequence), with q, k and v through z sigmoid(z)
//   pico_pair_close:  attention: the pieces of a column's keys put together, with its sink, gate and factor (as
//                     pico_attnb's second launch);  linear attention: norm over all heads and gate (as pico_gated_row_norm)
//
// Each of these launches is a chain of latencies a few microseconds long, and neither side waits for the other.
// Norms, angles, recurrence, state, softmax statistics and sums are float32.
#include "common.h"

#define PAIR_THREADS 256
#define PAIR_WAVES (PAIR_THREADS / 64)

struct OpenArgs {
  const bf16_t* x;              // [T, ld]
  int ld, T;
  // attention: columns of q, k, v; heads; sizes; rotation; where keys and values go
  int q_col, k_col, v_col, nq, nk, dk, dv, rot, P, num_pages, unit_wgs;
  float eps;
  const float* cos_sin;         // [T, rot / 2, 2]
  const int* slots;             // [T]
  bf16_t* q_out;
  bf16_t* k_cache;
  bf16_t* v_cache;
  // linear attention: columns of q, k, v; heads; sizes; a state slot a token
  int lq_col, lk_col, lv_col, H, ldk, ldv, num_slots, v_wgs;
  const int* state_slots;
  const float* decay;           // [H]
  float* state;                 // [slots, H, ldk, ldv]
  float* o;                     // [T, H ldv]
};

// Four query or key heads of a token, a wave each, and a part of its values.
__device__ __forceinline__ void open_attention(const OpenArgs& a, int wg) {
  const int t = wg / a.unit_wgs, part = wg % a.unit_wgs, lane = threadIdx.x & 63;
  const bf16_t* row = a.x + (size_t)t * a.ld;
  const int slot = a.slots[t];
  const int page = slot >= 0 ? slot / a.P : -1, off = slot >= 0 ? slot % a.P : 0;
  const bool store = page >= 0 && page < a.num_pages;
  const int u = part * PAIR_WAVES + (threadIdx.x >> 6);
  if (u < a.nq + a.nk) {
    const bool is_q = u < a.nq;
    const bf16_t* src = row + (is_q ? a.q_col + u * a.dk : a.k_col + (u - a.nq) * a.dk);
    float ss = 0.f;
    for (int i = lane; i < a.dk; i += 64) {
      const float v = bf16_to_f32(src[i]);
      ss = fmaf(v, v, ss);
    }
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)a.dk + a.eps);
    if (is_q || store) {
      bf16_t* dst = is_q ? a.q_out + ((size_t)t * a.nq + u) * a.dk : a.k_cache + (((size_t)page * a.nk + (u - a.nq)) * a.P + off) * a.dk;
      const float* cs = a.cos_sin + (size_t)t * a.rot;
      for (int i = lane; i < a.dk; i += 64) {
        float v = bf16_to_f32(src[i]) * r;
        if (i < a.rot) {
          const float w = bf16_to_f32(src[i ^ 1]) * r, c = cs[i & ~1], s = cs[i | 1];
          v = (i & 1) ? v * c + w * s : v * c - w * s;
        }
        dst[i] = f32_to_bf16(v);
      }
    }
  }
  if (store)
    for (int i = part * PAIR_THREADS + threadIdx.x; i < a.nk * a.dv; i += a.unit_wgs * PAIR_THREADS) {
      const int g = i / a.dv, j = i % a.dv;
      a.v_cache[(((size_t)page * a.nk + g) * a.dv + j) * a.P + off] = row[a.v_col + i];
    }
}

// One head of a token and 64 of its value channels, a lane each; the waves share the key channels and meet in LDS.
#define PAIR_AHEAD 16            // elements of the state a lane asks for at a time
#define PAIR_MAX_KEY 256
__device__ __forceinline__ void open_linear(const OpenArgs& a, int wg) {
  __shared__ float qs[PAIR_MAX_KEY], ks[PAIR_MAX_KEY], part[PAIR_WAVES][64];
  const int vb = wg % a.v_wgs, h = wg / a.v_wgs % a.H, t = wg / (a.v_wgs * a.H), lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int slot = a.state_slots[t];
  if (slot < 0 || slot >= a.num_slots) return;                          // the whole workgroup
  const bf16_t* row = a.x + (size_t)t * a.ld;
  const int v = vb * 64 + lane, v_in = min(v, a.ldv - 1);
  const int each = (a.ldk + PAIR_WAVES - 1) / PAIR_WAVES, c0 = wave * each, c1 = min(a.ldk, c0 + each);
  float* sp = a.state + ((size_t)slot * a.H + h) * a.ldk * a.ldv + v_in;
  float S[PAIR_AHEAD];
#pragma unroll
  for (int i = 0; i < PAIR_AHEAD; i++) S[i] = sp[(size_t)min(c0 + i, a.ldk - 1) * a.ldv];
  const float vv = silu_f(bf16_to_f32(row[a.lv_col + h * a.ldv + v_in])), g = a.decay[h];
  for (int c = threadIdx.x; c < a.ldk; c += PAIR_THREADS) {
    qs[c] = silu_f(bf16_to_f32(row[a.lq_col + h * a.ldk + c]));
    ks[c] = silu_f(bf16_to_f32(row[a.lk_col + h * a.ldk + c]));
  }
  __syncthreads();
  float acc = 0.f;
  for (int b = c0; b < c1; b += PAIR_AHEAD) {
    if (b > c0) {
#pragma unroll
      for (int i = 0; i < PAIR_AHEAD; i++) S[i] = sp[(size_t)min(b + i, a.ldk - 1) * a.ldv];
    }
#pragma unroll
    for (int i = 0; i < PAIR_AHEAD; i++) {
      const int c = min(b + i, a.ldk - 1);
      const float s = fmaf(g, S[i], ks[c] * vv);
      if (b + i < c1) {
        acc = fmaf(s, qs[c], acc);
        if (v < a.ldv) sp[(size_t)c * a.ldv] = s;
      }
    }
  }
  part[wave][lane] = acc;
  __syncthreads();
  if (wave == 0 && v < a.ldv) {
    float sum = part[0][lane];
#pragma unroll
    for (int w = 1; w < PAIR_WAVES; w++) sum += part[w][lane];
    a.o[((size_t)t * a.H + h) * a.ldv + v] = sum;
  }
}

// workgroups: the linear attention's first (they take longer)
__global__ __launch_bounds__(PAIR_THREADS) void pair_open_kernel(const OpenArgs a) {
  const int linear = a.T * a.H * a.v_wgs, wg = blockIdx.x;
  if (wg < linear) open_linear(a, wg);
  else open_attention(a, wg - linear);
}

extern "C" int pico_pair_open(const void* x, int ld, int T, int q_col, int k_col, int v_col, int nq, int nk, int dk, int dv, int rot,
                              float eps, const float* cos_sin, const int* slots, void* q_out, void* k_cache, void* v_cache, int P,
                              int num_pages, int lq_col, int lk_col, int lv_col, int H, int ldk, int ldv, const int* state_slots,
                              const float* decay, float* state, float* o, int num_slots, hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && nq > 0 && nk > 0 && dk > 0 && dv > 0 && P > 0 && num_pages > 0 && H > 0 && ldk > 0 && ldv > 0 && num_slots > 0,
               "pico_pair_open: bad sizes");
  PICO_REQUIRE(ldk <= PAIR_MAX_KEY, "pico_pair_open: at most %d key channels a head, got %d", PAIR_MAX_KEY, ldk);
  PICO_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= dk && (rot == 0 || cos_sin), "pico_pair_open: %d turned entries of %d", rot, dk);
  PICO_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && lq_col >= 0 && lk_col >= 0 && lv_col >= 0 && ld >= q_col + nq * dk &&
                   ld >= k_col + nk * dk && ld >= v_col + nk * dv && ld >= lq_col + H * ldk && ld >= lk_col + H * ldk && ld >= lv_col + H * ldv,
               "pico_pair_open: the row of %d columns does not hold both sides", ld);
  PICO_REQUIRE(slots && q_out && k_cache && v_cache && state_slots && decay && state && o, "pico_pair_open: a tensor is missing");
  if (T == 0) return 0;
  const int unit_wgs = (nq + nk + PAIR_WAVES - 1) / PAIR_WAVES, v_wgs = (ldv + 63) / 64;
  const long long wgs = (long long)T * (unit_wgs + (long long)H * v_wgs);
  PICO_REQUIRE(wgs < (1ll << 31), "pico_pair_open: sizes beyond the grid");
  const OpenArgs a{(const bf16_t*)x, ld, T, q_col, k_col, v_col, nq, nk, dk, dv, rot, P, num_pages, unit_wgs, eps, cos_sin, slots, (bf16_t*)q_out,
                   (bf16_t*)k_cache, (bf16_t*)v_cache, lq_col, lk_col, lv_col, H, ldk, ldv, num_slots, v_wgs, state_slots, decay, state, o};
  pair_open_kernel<<<(unsigned)wgs, PAIR_THREADS, 0, stream>>>(a);
  PICO_LAUNCH_CHECK();
  return 0;
}

struct CloseArgs {
  int T;
  // attention: pieces of every (token, head) column
  const float* parts_o;         // [pieces, T nq, dv], unnormalised
  const float* parts_ml;        // [pieces, T nq, 2]: maximum, sum
  int pieces, nq, dv;
  const float* sinks;           // [nq]
  const bf16_t* gate;           // [T, >= nq]
  int gate_stride;
  float out_scale;
  bf16_t* out;                  // rows out_stride apart
  int out_stride;
  // linear attention: rows of N
  const float* o;
  const bf16_t* lgate;
  int lgate_stride, N;
  const float* w;
  float eps;
  bf16_t* lout;
  int lout_stride;
};

#define CLOSE_THREADS 1024
#define CLOSE_VPT 4
#define CLOSE_MAX_PIECES 64
#define CLOSE_MAX_DV 256

// A column a group of CLOSE_WAVES waves: lane z of each holds piece z's maximum and sum; a wave takes every CLOSE_WAVES-th
// piece, CLOSE_AHEAD of them at a time for 128 value entries (two a lane), and the waves meet in LDS.
#define CLOSE_WAVES 4
#define CLOSE_COLS (CLOSE_THREADS / 64 / CLOSE_WAVES)
#define CLOSE_AHEAD 8
__device__ __forceinline__ void close_attention(const CloseArgs& a, int wg) {
  __shared__ float sums[CLOSE_THREADS / 64][128];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, sub = wave % CLOSE_WAVES, ncols = a.T * a.nq;
  const int mine = wg * CLOSE_COLS + wave / CLOSE_WAVES, c = min(mine, ncols - 1);
  const int t = c / a.nq, h = c % a.nq;
  float2 ml = *reinterpret_cast<const float2*>(a.parts_ml + 2 * ((size_t)min(lane, a.pieces - 1) * ncols + c));
  if (lane >= a.pieces) ml = make_float2(-INFINITY, 0.f);
  const float sink = a.sinks[h], gate = bf16_to_f32(a.gate[(size_t)t * a.gate_stride + h]);
  const size_t step = (size_t)ncols * a.dv;
  for (int d0 = 0; d0 < a.dv; d0 += 128) {
    const float* p0 = a.parts_o + (size_t)c * a.dv + min(d0 + lane, a.dv - 1);
    const float* p1 = a.parts_o + (size_t)c * a.dv + min(d0 + 64 + lane, a.dv - 1);
    float acc0 = 0.f, acc1 = 0.f, M, w;
    for (int z0 = sub; z0 < a.pieces; z0 += CLOSE_WAVES * CLOSE_AHEAD) {
      float v0[CLOSE_AHEAD], v1[CLOSE_AHEAD];
#pragma unroll
      for (int i = 0; i < CLOSE_AHEAD; i++) {
        const size_t z = min(z0 + CLOSE_WAVES * i, a.pieces - 1);
        v0[i] = p0[z * step];
        v1[i] = p1[z * step];
      }
      M = wave_max(ml.x);
      w = ml.x == -INFINITY ? 0.f : __expf(ml.x - M);
#pragma unroll
      for (int i = 0; i < CLOSE_AHEAD; i++) {
        const int z = z0 + CLOSE_WAVES * i;
        const float wz = z < a.pieces ? __shfl(w, min(z, 63)) : 0.f;
        acc0 = fmaf(v0[i], wz, acc0);
        acc1 = fmaf(v1[i], wz, acc1);
      }
    }
    __syncthreads();                                     // the last 128 entries' sums have been read
    sums[wave][lane] = acc0;
    sums[wave][64 + lane] = acc1;
    __syncthreads();
    // entry 32 sub + lane (of 128): a quarter a wave
    M = wave_max(ml.x);
    w = ml.x == -INFINITY ? 0.f : __expf(ml.x - M);
    // (the column's own key is always seen: M is finite.  A sink so far above every key that its exponential overflows
    // leaves the keys no weight)
    const float L = wave_sum(ml.y * w) + __expf(sink - M);
    const float f = a.out_scale / L / (1.0f + __expf(-gate));
    const int e = 32 * sub + (lane & 31), first = wave - sub;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < CLOSE_WAVES; i++) sum += sums[first + i][e];
    if (lane < 32 && mine < ncols && d0 + e < a.dv) a.out[(size_t)t * a.out_stride + h * a.dv + d0 + e] = f32_to_bf16(sum * f);
  }
}

__device__ __forceinline__ void close_linear(const CloseArgs& a, int t) {
  __shared__ float scratch[16];
  float v[CLOSE_VPT], g[CLOSE_VPT], w[CLOSE_VPT];
#pragma unroll
  for (int j = 0; j < CLOSE_VPT; j++) {
    const int i = min(j * CLOSE_THREADS + (int)threadIdx.x, a.N - 1);
    v[j] = a.o[(size_t)t * a.N + i];
    g[j] = bf16_to_f32(a.lgate[(size_t)t * a.lgate_stride + i]);
    w[j] = a.w[i];
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < CLOSE_VPT; j++)
    if (j * CLOSE_THREADS + (int)threadIdx.x < a.N) ss = fmaf(v[j], v[j], ss);
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)a.N + a.eps);
#pragma unroll
  for (int j = 0; j < CLOSE_VPT; j++) {
    const int i = j * CLOSE_THREADS + (int)threadIdx.x;
    if (i < a.N) a.lout[(size_t)t * a.lout_stride + i] = f32_to_bf16(v[j] * r * w[j] / (1.0f + expf(-g[j])));
  }
}

__global__ __launch_bounds__(CLOSE_THREADS) void pair_close_kernel(const CloseArgs a) {
  if ((int)blockIdx.x < a.T) close_linear(a, blockIdx.x);
  else close_attention(a, blockIdx.x - a.T);
}

extern "C" int pico_pair_close(int T, const float* parts_o, const float* parts_ml, int pieces, int nq, int dv, const float* sinks,
                               const void* gate, int gate_stride, float out_scale, void* out, int out_stride, const float* o,
                               const void* lgate, int lgate_stride, int N, const float* w, float eps, void* lout, int lout_stride,
                               hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && nq > 0 && dv > 0 && dv <= CLOSE_MAX_DV && pieces >= 1 && pieces <= CLOSE_MAX_PIECES, "pico_pair_close: bad sizes");
  PICO_REQUIRE(N > 0 && N <= CLOSE_THREADS * CLOSE_VPT && eps > 0.f, "pico_pair_close: rows of 1 to %d entries, got %d", CLOSE_THREADS * CLOSE_VPT, N);
  PICO_REQUIRE(gate_stride >= nq && out_stride >= nq * dv && lgate_stride >= N && lout_stride >= N, "pico_pair_close: row strides too small");
  PICO_REQUIRE(parts_o && parts_ml && sinks && gate && out && o && lgate && w && lout && (uintptr_t)parts_ml % 8 == 0, "pico_pair_close: bad operands");
  if (T == 0) return 0;
  const long long wgs = T + ((long long)T * nq + CLOSE_COLS - 1) / CLOSE_COLS;
  PICO_REQUIRE(wgs < (1ll << 31), "pico_pair_close: sizes beyond the grid");
  const CloseArgs a{T, parts_o, parts_ml, pieces, nq, dv, sinks, (const bf16_t*)gate, gate_stride, out_scale, (bf16_t*)out, out_stride, o,
                    (const bf16_t*)lgate, lgate_stride, N, w, eps, (bf16_t*)lout, lout_stride};
  pair_close_kernel<<<(unsigned)wgs, CLOSE_THREADS, 0, stream>>>(a);
  PICO_LAUNCH_CHECK();
  return 0;
}
