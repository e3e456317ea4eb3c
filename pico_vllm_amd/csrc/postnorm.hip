// Norms of a layer that norms what a sublayer RETURNS (x <- x + norm(sublayer(x))), and of the stream itself.
//
//   pico_norm_add:        x[t] += rms(y[t]) * w                          (y: the sublayer's output)
//                         or, with two outputs a and b and a weight each,
//                         x[t] += rms( (rms(a[t]) * wa + rms(b[t]) * wb) / 2 ) * w
//   pico_norm_add_norm:   x[t] += rms(y[t]) * w (+ a vector, the same for every row), and out[t] = rms(x[t]) * w_next (the next
//                         sublayer's norm in front of it) or, without w_next, x[t] itself in the activations' storage type
//   pico_stream_rmsnorm:  x[t] <- rms(x[t]) * w
//   rms(v) = v / sqrt(mean(v^2) + eps).  Both can leave a copy of the new x in the activations' storage type, which is
//   what the next sublayer reads.
//
// x is the float32 residual stream.  An output may be [T, H] in float32 or bfloat16, or a float32 stack [S, T, H] of
// partial sums of the product that made it, which are added up first (in the order of the stack).  All arithmetic is
// float32; a row's sums run in an order that depends on H alone.  One workgroup a row, the row kept in LDS.
#include "common.h"

#define POSTNORM_MAX_SLABS 8

// The slabs' entries added up in the order of the stack; all loads are issued before the first sum waits for one.
template <typename T>
__device__ __forceinline__ float summed(const T* __restrict__ y, int slabs, size_t slab_stride, size_t at) {
  float part[POSTNORM_MAX_SLABS];
#pragma unroll
  for (int s = 0; s < POSTNORM_MAX_SLABS; s++) part[s] = load_f32(y + (size_t)min(s, slabs - 1) * slab_stride + at);
  float v = part[0];
#pragma unroll
  for (int s = 1; s < POSTNORM_MAX_SLABS; s++) v += s < slabs ? part[s] : 0.f;
  return v;
}

// TA, TB: the types of a and b; TO: the type of the copy.
template <typename TA, typename TB, typename TO>
__global__ __launch_bounds__(1024) void norm_add_kernel(float* __restrict__ x, const TA* __restrict__ a, int a_slabs,
                                                       const float* __restrict__ wa, const TB* __restrict__ b, int b_slabs,
                                                       const float* __restrict__ wb, size_t slab_stride,
                                                       const float* __restrict__ w, float eps, TO* __restrict__ copy, int H) {
  extern __shared__ float row[];          // [H] (and [H] more with b)
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const size_t base = (size_t)t * H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = summed(a, a_slabs, slab_stride, base + i);
    row[i] = v;
    ss = fmaf(v, v, ss);
  }
  const float ra = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
  if (b) {
    float* rb_row = row + H;
    float sb = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
      const float v = summed(b, b_slabs, slab_stride, base + i);
      rb_row[i] = v;
      sb = fmaf(v, v, sb);
    }
    const float rb = 1.0f / sqrtf(block_sum(sb, scratch) / (float)H + eps);
    float sm = 0.f;
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
      const float v = 0.5f * (row[i] * ra * wa[i] + rb_row[i] * rb * wb[i]);
      row[i] = v;
      sm = fmaf(v, v, sm);
    }
    const float rm = 1.0f / sqrtf(block_sum(sm, scratch) / (float)H + eps);
    for (int i = threadIdx.x; i < H; i += blockDim.x) {
      const float v = x[base + i] + row[i] * rm * w[i];
      x[base + i] = v;
      if (copy) store_f32(copy + base + i, v);
    }
    return;
  }
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = x[base + i] + row[i] * ra * w[i];
    x[base + i] = v;
    if (copy) store_f32(copy + base + i, v);
  }
}

// V neighbouring entries
template <typename T, int V> __device__ __forceinline__ void load_v(const T* p, float* v) {
  if constexpr (V == 1) {
    v[0] = load_f32(p);
  } else if constexpr (sizeof(T) == 4) {
    const float4 r = *reinterpret_cast<const float4*>(p);
    v[0] = r.x; v[1] = r.y; v[2] = r.z; v[3] = r.w;
  } else {
    const uint2 r = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(r.x << 16); v[1] = __uint_as_float(r.x & 0xffff0000u);
    v[2] = __uint_as_float(r.y << 16); v[3] = __uint_as_float(r.y & 0xffff0000u);
  }
}
template <typename T, int V> __device__ __forceinline__ void store_v(T* p, const float* v) {
  if constexpr (V == 1) store_f32(p, v[0]);
  else if constexpr (sizeof(T) == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(v[0], v[1]), pack2_bf16(v[2], v[3]));
}

// Norm of the output, sum and norm of the sum with the row in registers: a thread owns VPT times V neighbouring entries,
// thread i the entries (j * blockDim + i) * V ..; the number of threads goes with H alone, so a row's sums run in one order
// whatever stands beside it.  All loads of a row are issued before the first sum.
template <typename TY, typename TO, int V, int VPT>
__global__ __launch_bounds__(1024) void norm_add_norm_kernel(float* __restrict__ x, const TY* __restrict__ y, int slabs,
                                                             size_t slab_stride, const float* __restrict__ w, float eps,
                                                             const float* __restrict__ w_next, float eps_next, TO* __restrict__ out,
                                                             int ld_out, int H, const float* __restrict__ vec) {
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * H;
  float yv[VPT][V], xv[VPT][V], wv[VPT][V];
  bool ok[VPT];
#pragma unroll
  for (int j = 0; j < VPT; j++) {
    const int at = (j * (int)blockDim.x + (int)threadIdx.x) * V;
    ok[j] = at < H;
    const int i = ok[j] ? at : 0;
    load_v<float, V>(x + base + i, xv[j]);
    load_v<float, V>(w + i, wv[j]);
    load_v<TY, V>(y + base + i, yv[j]);
  }
  for (int s = 1; s < slabs; s++) {
    float more[VPT][V];
#pragma unroll
    for (int j = 0; j < VPT; j++) load_v<TY, V>(y + s * slab_stride + base + (ok[j] ? (j * (int)blockDim.x + (int)threadIdx.x) * V : 0), more[j]);
#pragma unroll
    for (int j = 0; j < VPT; j++)
#pragma unroll
      for (int k = 0; k < V; k++) yv[j][k] += more[j][k];
  }
  float add[VPT][V];
  if (vec) {
#pragma unroll
    for (int j = 0; j < VPT; j++) load_v<float, V>(vec + (ok[j] ? (j * (int)blockDim.x + (int)threadIdx.x) * V : 0), add[j]);
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < VPT; j++)
#pragma unroll
    for (int k = 0; k < V; k++) ss = ok[j] ? fmaf(yv[j][k], yv[j][k], ss) : ss;
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
  ss = 0.f;
#pragma unroll
  for (int j = 0; j < VPT; j++) {
#pragma unroll
    for (int k = 0; k < V; k++) {
      xv[j][k] += yv[j][k] * r * wv[j][k];
      if (vec) xv[j][k] += add[j][k];
      ss = ok[j] ? fmaf(xv[j][k], xv[j][k], ss) : ss;
    }
    if (ok[j]) store_v<float, V>(x + base + (j * (int)blockDim.x + (int)threadIdx.x) * V, xv[j]);
  }
  if (out == nullptr) return;
  if (w_next) {
#pragma unroll
    for (int j = 0; j < VPT; j++) load_v<float, V>(w_next + (ok[j] ? (j * (int)blockDim.x + (int)threadIdx.x) * V : 0), wv[j]);
    const float rn = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps_next);
#pragma unroll
    for (int j = 0; j < VPT; j++)
#pragma unroll
      for (int k = 0; k < V; k++) xv[j][k] *= rn * wv[j][k];
  }
#pragma unroll
  for (int j = 0; j < VPT; j++)
    if (ok[j]) store_v<TO, V>(out + (size_t)blockIdx.x * ld_out + (j * (int)blockDim.x + (int)threadIdx.x) * V, xv[j]);
}

template <typename TO>
__global__ __launch_bounds__(256) void stream_rmsnorm_kernel(float* __restrict__ x, const float* __restrict__ w, float eps,
                                                             TO* __restrict__ copy, int H) {
  extern __shared__ float row[];
  __shared__ float scratch[16];
  const size_t base = (size_t)blockIdx.x * H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = x[base + i];
    row[i] = v;
    ss = fmaf(v, v, ss);
  }
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = row[i] * r * w[i];
    x[base + i] = v;
    if (copy) store_f32(copy + base + i, v);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void cast_rows_kernel(const float* __restrict__ x, T* __restrict__ out, long long n) {
  const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) store_f32(out + i, x[i]);
}

#define POSTNORM_MAX_H 16384     // floats of LDS a workgroup may ask for (64 KB)

extern "C" int pico_norm_add(float* x, const void* a, int a_dtype, int a_slabs, const float* wa, const void* b, int b_dtype,
                             int b_slabs, const float* wb, long long slab_stride, const float* w, float eps, void* copy, int copy_dtype,
                             int T, int H, hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && H > 0 && H * (b ? 2 : 1) <= POSTNORM_MAX_H, "pico_norm_add: a width of 1 to %d (half with two outputs), got %d", POSTNORM_MAX_H, H);
  PICO_REQUIRE(a != nullptr && a_slabs >= 1 && (b == nullptr || (b_slabs >= 1 && wa && wb)), "pico_norm_add: bad operands");
  PICO_REQUIRE(a_slabs <= POSTNORM_MAX_SLABS && b_slabs <= POSTNORM_MAX_SLABS, "pico_norm_add: at most %d partial sums an output", POSTNORM_MAX_SLABS);
  PICO_REQUIRE((a_slabs == 1 || a_dtype == PICO_DTYPE_F32) && (b == nullptr || b_slabs == 1 || b_dtype == PICO_DTYPE_F32),
               "pico_norm_add: partial sums are float32");
  if (b == nullptr) b_dtype = a_dtype;
  if (copy == nullptr) copy_dtype = PICO_DTYPE_F32;
  if (T == 0) return 0;
  const size_t lds = (size_t)H * sizeof(float) * (b ? 2 : 1);
  // few rows: as many threads as the row has entries (up to 1,024), so that a thread's loads are one turn and travel
  // together; many rows fill the chip with four waves each
  const int threads = T >= 64 ? 256 : min(1024, max(256, (H + 63) / 64 * 64));
#define LAUNCH(TA, TB, TO)                                                                                                   \
  norm_add_kernel<TA, TB, TO><<<T, threads, lds, stream>>>(x, (const TA*)a, a_slabs, wa, (const TB*)b, b_slabs, wb,              \
                                                       (size_t)slab_stride, w, eps, (TO*)copy, H)
  const int key = (a_dtype == PICO_DTYPE_BF16 ? 4 : 0) | (b_dtype == PICO_DTYPE_BF16 ? 2 : 0) | (copy_dtype == PICO_DTYPE_BF16 ? 1 : 0);
  PICO_REQUIRE((a_dtype | 1) == 1 && (b_dtype | 1) == 1 && (copy_dtype | 1) == 1, "pico_norm_add: unknown dtype");
  switch (key) {
    case 0: LAUNCH(float, float, float); break;
    case 1: LAUNCH(float, float, bf16_t); break;
    case 2: LAUNCH(float, bf16_t, float); break;
    case 3: LAUNCH(float, bf16_t, bf16_t); break;
    case 4: LAUNCH(bf16_t, float, float); break;
    case 5: LAUNCH(bf16_t, float, bf16_t); break;
    case 6: LAUNCH(bf16_t, bf16_t, float); break;
    default: LAUNCH(bf16_t, bf16_t, bf16_t); break;
  }
#undef LAUNCH
  PICO_LAUNCH_CHECK();
  return 0;
}

extern "C" int pico_norm_add_norm(float* x, const void* y, int y_dtype, int slabs, long long slab_stride, const float* w, float eps,
                                  const float* w_next, float eps_next, void* out, int out_dtype, int ld_out, int T, int H,
                                  const float* vec, hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && H > 0 && H <= POSTNORM_MAX_H, "pico_norm_add_norm: a width of 1 to %d, got %d", POSTNORM_MAX_H, H);
  PICO_REQUIRE(x && y && w && slabs >= 1 && (slabs == 1 || y_dtype == PICO_DTYPE_F32), "pico_norm_add_norm: bad operands (partial sums are float32)");
  PICO_REQUIRE(eps > 0.f && (w_next == nullptr || (eps_next > 0.f && out)) && (out == nullptr || ld_out >= H), "pico_norm_add_norm: bad operands");
  PICO_REQUIRE((y_dtype | 1) == 1 && (out_dtype | 1) == 1, "pico_norm_add_norm: unknown dtype");
  if (T == 0) return 0;
  const uintptr_t all = (uintptr_t)x | (uintptr_t)y | (uintptr_t)w | (uintptr_t)w_next | (uintptr_t)out | (uintptr_t)vec;
  // (every pointer on 16 bytes and rows of whole fours: then so is every row, or on 8 bytes where storage is bfloat16)
  const bool four = H % 4 == 0 && all % 16 == 0 && (out == nullptr || ld_out % 4 == 0) && (slabs == 1 || slab_stride % 4 == 0);
  const int units = four ? H / 4 : H;
  const int vpt = units <= 1024 ? 1 : units <= 4096 ? 4 : 16;
  const int threads = ((units + vpt - 1) / vpt + 63) / 64 * 64;
#define LAUNCH(TY, TO, V, VPT)                                                                                                   \
  norm_add_norm_kernel<TY, TO, V, VPT><<<T, threads, 0, stream>>>(x, (const TY*)y, slabs, (size_t)slab_stride, w, eps, w_next,   \
                                                                  eps_next, (TO*)out, ld_out, H, vec)
#define PICK(TY, TO)                              \
  do {                                            \
    if (four && vpt == 1) LAUNCH(TY, TO, 4, 1);   \
    else if (four) LAUNCH(TY, TO, 4, 4);          \
    else if (vpt == 1) LAUNCH(TY, TO, 1, 1);      \
    else if (vpt == 4) LAUNCH(TY, TO, 1, 4);      \
    else LAUNCH(TY, TO, 1, 16);                   \
  } while (0)
  if (y_dtype == PICO_DTYPE_F32) {
    if (out_dtype == PICO_DTYPE_F32) PICK(float, float); else PICK(float, bf16_t);
  } else {
    if (out_dtype == PICO_DTYPE_F32) PICK(bf16_t, float); else PICK(bf16_t, bf16_t);
  }
#undef PICK
#undef LAUNCH
  PICO_LAUNCH_CHECK();
  return 0;
}

// out[t][i] = x[t][i] in the storage type `dtype`; rows of the output lie ld_out apart.
template <typename T>
__global__ __launch_bounds__(256) void store_rows_kernel(const float* __restrict__ x, T* __restrict__ out, int ld_out, int H) {
  for (int i = threadIdx.x; i < H; i += blockDim.x) store_f32(out + (size_t)blockIdx.x * ld_out + i, x[(size_t)blockIdx.x * H + i]);
}

extern "C" int pico_store_rows(const float* x, void* out, int dtype, int ld_out, int T, int H, hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && H > 0 && ld_out >= H, "pico_store_rows: bad sizes");
  if (T == 0) return 0;
  if (dtype == PICO_DTYPE_F32) store_rows_kernel<float><<<T, 256, 0, stream>>>(x, (float*)out, ld_out, H);
  else if (dtype == PICO_DTYPE_BF16) store_rows_kernel<bf16_t><<<T, 256, 0, stream>>>(x, (bf16_t*)out, ld_out, H);
  else PICO_REQUIRE(false, "pico_store_rows: unknown dtype %d", dtype);
  PICO_LAUNCH_CHECK();
  return 0;
}

extern "C" int pico_stream_rmsnorm(float* x, const float* w, float eps, void* copy, int copy_dtype, int T, int H,
                                   hipStream_t stream) {
  PICO_REQUIRE(T >= 0 && H > 0 && H <= POSTNORM_MAX_H, "pico_stream_rmsnorm: a width of 1 to %d, got %d", POSTNORM_MAX_H, H);
  if (T == 0) return 0;
  const size_t lds = (size_t)H * sizeof(float);
  if (copy == nullptr || copy_dtype == PICO_DTYPE_F32)
    stream_rmsnorm_kernel<float><<<T, 256, lds, stream>>>(x, w, eps, (float*)copy, H);
  else if (copy_dtype == PICO_DTYPE_BF16)
    stream_rmsnorm_kernel<bf16_t><<<T, 256, lds, stream>>>(x, w, eps, (bf16_t*)copy, H);
  else
    PICO_REQUIRE(false, "pico_stream_rmsnorm: unknown dtype %d", copy_dtype);
  PICO_LAUNCH_CHECK();
  return 0;
}

extern "C" int pico_cast_rows(const float* x, void* out, int dtype, long long n, hipStream_t stream) {
  PICO_REQUIRE(n >= 0 && dtype == PICO_DTYPE_BF16, "pico_cast_rows: float32 to bfloat16 only");
  if (n == 0) return 0;
  cast_rows_kernel<bf16_t><<<(unsigned)((n + 255) / 256), 256, 0, stream>>>(x, (bf16_t*)out, n);
  PICO_LAUNCH_CHECK();
  return 0;
}
