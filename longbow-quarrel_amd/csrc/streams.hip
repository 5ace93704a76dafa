// Hyper-connections: a residual of several streams between the sublayers of a decoder (`lq_streams_step`), and the
// soft cap on the logits.  Everything is 32-bit; only what the next matrix product reads is rounded to the run's dtype.
#include "common.h"

namespace {

// One row of the step:
//   Y = the sum of the sublayer's pieces;   X'_t = sum_s mix[s, t] X_s + out[t] Y      (y given: the streams are written)
//   u = sum_t read[t] X'_t (read null: the plain sum);   h = u / sqrt(mean(u^2) + eps) * w         (h given)
// With no y the streams are only read (X' = X).  `src_stride` 0: one stored stream stands for all (the start of a
// sequence of layers, where they are equal).  src and dst may be the same streams: a thread reads its entries of all of
// them before it writes any.  Sums over streams and pieces go in ascending order, the sum of squares is the block's fixed
// tree: a row's result depends on the row alone.
struct StreamArgs {
  const float* src;
  long long src_stride;  // floats from stream to stream
  float* dst;            // [S][rows][width]
  long long dst_stride;
  const float* y;  // [pieces][rows][width], or null
  int pieces;
  long long y_stride;
  const float *mix, *out_w, *read_w, *norm_w;
  float eps;
  int S, width;
};

constexpr int MAX_STREAMS = 16;

// Rows of up to 256 * 4 * KEEP entries in fours, all rows on 16 bytes: what the norm reads (u) stays in registers, so a
// row is read once.  NS: the number of streams, 0: a.S of them.
template <typename T, int NS, int KEEP>
__global__ __launch_bounds__(256) void streams_step4_kernel(StreamArgs a, T* __restrict__ h) {
  __shared__ float red[16];
  const int S = NS > 0 ? NS : a.S;
  constexpr int XS = NS > 0 ? NS : MAX_STREAMS;
  // the weights are the same for all threads: read once, ahead of all stores (a known few of them into scalar registers)
  __shared__ float mix_lds[NS > 0 ? 1 : MAX_STREAMS * MAX_STREAMS];
  float mix_own[NS > 0 ? NS * NS : 1], out_w[XS], read_w[XS];
  if constexpr (NS > 0) {
#pragma unroll
    for (int i = 0; i < NS * NS; ++i) mix_own[i] = a.y != nullptr ? a.mix[i] : 0.f;
  } else {
    for (int i = threadIdx.x; i < S * S; i += 256) mix_lds[i] = a.y != nullptr ? a.mix[i] : 0.f;
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < XS; ++t) {
    out_w[t] = a.y != nullptr && t < S ? a.out_w[t] : 0.f;
    read_w[t] = a.read_w != nullptr && t < S ? a.read_w[t] : 1.f;
  }
  auto mix = [&](int s, int t) { return NS > 0 ? mix_own[NS > 0 ? s * NS + t : 0] : mix_lds[NS > 0 ? 0 : s * S + t]; };
  const long long base = (long long)blockIdx.x * a.width;
  const int n4 = a.width >> 2;
  float4 u[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < KEEP; ++j) {
    const int i = threadIdx.x + j * 256;
    u[j] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (i >= n4) continue;
    float4 x[XS];
#pragma unroll
    for (int s = 0; s < XS; ++s)
      if (s < S) x[s] = reinterpret_cast<const float4*>(a.src + s * a.src_stride + base)[i];
    if (a.y != nullptr) {
      float4 y = reinterpret_cast<const float4*>(a.y + base)[i];
      for (int p = 1; p < a.pieces; ++p) {
        const float4 b = reinterpret_cast<const float4*>(a.y + p * a.y_stride + base)[i];
        y.x += b.x, y.y += b.y, y.z += b.z, y.w += b.w;
      }
#pragma unroll
      for (int t = 0; t < XS; ++t) {
        if (t >= S) continue;
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < XS; ++s)
          if (s < S) {
            const float m = mix(s, t);
            v.x = fmaf(m, x[s].x, v.x), v.y = fmaf(m, x[s].y, v.y), v.z = fmaf(m, x[s].z, v.z), v.w = fmaf(m, x[s].w, v.w);
          }
        const float o = out_w[t], r = read_w[t];
        v.x = fmaf(o, y.x, v.x), v.y = fmaf(o, y.y, v.y), v.z = fmaf(o, y.z, v.z), v.w = fmaf(o, y.w, v.w);
        reinterpret_cast<float4*>(a.dst + t * a.dst_stride + base)[i] = v;
        u[j].x = fmaf(r, v.x, u[j].x), u[j].y = fmaf(r, v.y, u[j].y), u[j].z = fmaf(r, v.z, u[j].z), u[j].w = fmaf(r, v.w, u[j].w);
      }
    } else {
#pragma unroll
      for (int t = 0; t < XS; ++t)
        if (t < S) {
          const float r = read_w[t];
          u[j].x = fmaf(r, x[t].x, u[j].x), u[j].y = fmaf(r, x[t].y, u[j].y);
          u[j].z = fmaf(r, x[t].z, u[j].z), u[j].w = fmaf(r, x[t].w, u[j].w);
        }
    }
    ss = fmaf(u[j].x, u[j].x, fmaf(u[j].y, u[j].y, fmaf(u[j].z, u[j].z, fmaf(u[j].w, u[j].w, ss))));
  }
  if (h == nullptr) return;
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.width + a.eps);
#pragma unroll
  for (int j = 0; j < KEEP; ++j) {
    const int i = threadIdx.x + j * 256;
    if (i >= n4) continue;
    const float4 w = reinterpret_cast<const float4*>(a.norm_w)[i];
    const float y0 = u[j].x * inv * w.x, y1 = u[j].y * inv * w.y, y2 = u[j].z * inv * w.z, y3 = u[j].w * inv * w.w;
    T* o = h + base + 4 * (long long)i;
    if constexpr (sizeof(T) == 4) {
      *(float4*)o = make_float4(y0, y1, y2, y3);
    } else {
      uint2 packed;
      packed.x = (uint32_t)f32_to_bf16(y0).bits | ((uint32_t)f32_to_bf16(y1).bits << 16);
      packed.y = (uint32_t)f32_to_bf16(y2).bits | ((uint32_t)f32_to_bf16(y3).bits << 16);
      *(uint2*)o = packed;
    }
  }
}

// Any width: entry by entry, u made again from the written streams for the norm.
template <typename T>
__global__ __launch_bounds__(256) void streams_step_kernel(StreamArgs a, T* __restrict__ h) {
  __shared__ float red[16];
  const int S = a.S;
  const long long base = (long long)blockIdx.x * a.width;
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.width; i += 256) {
    float u = 0.f;
    if (a.y != nullptr) {
      float x[MAX_STREAMS];
#pragma unroll
      for (int s = 0; s < MAX_STREAMS; ++s) x[s] = s < S ? a.src[s * a.src_stride + base + i] : 0.f;
      float y = a.y[base + i];
      for (int p = 1; p < a.pieces; ++p) y += a.y[p * a.y_stride + base + i];
      for (int t = 0; t < S; ++t) {
        float v = 0.f;
#pragma unroll
        for (int s = 0; s < MAX_STREAMS; ++s)
          if (s < S) v = fmaf(a.mix[s * S + t], x[s], v);
        v = fmaf(a.out_w[t], y, v);
        a.dst[t * a.dst_stride + base + i] = v;
        u = fmaf(a.read_w != nullptr ? a.read_w[t] : 1.f, v, u);
      }
    } else {
      for (int t = 0; t < S; ++t) u = fmaf(a.read_w != nullptr ? a.read_w[t] : 1.f, a.src[t * a.src_stride + base + i], u);
    }
    ss = fmaf(u, u, ss);
  }
  if (h == nullptr) return;
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.width + a.eps);
  const float* from = a.y != nullptr ? a.dst : a.src;  // (a thread reads back the entries that it wrote)
  const long long stride = a.y != nullptr ? a.dst_stride : a.src_stride;
  for (int i = threadIdx.x; i < a.width; i += 256) {
    float u = 0.f;
    for (int t = 0; t < S; ++t) u = fmaf(a.read_w != nullptr ? a.read_w[t] : 1.f, from[t * stride + base + i], u);
    h[base + i] = from_f32<T>(u * inv * a.norm_w[i]);
  }
}

// x <- cap tanh(x factor / cap)
__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ x, float cap, float factor, long long n) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] * factor / cap);
}

template <typename T, int NS>
void launch_streams4(const StreamArgs& a, T* h, int rows, hipStream_t stream) {
  const int n4 = a.width / 4;
  if (n4 <= 256) streams_step4_kernel<T, NS, 1><<<rows, 256, 0, stream>>>(a, h);
  else if (n4 <= 512) streams_step4_kernel<T, NS, 2><<<rows, 256, 0, stream>>>(a, h);
  else if (n4 <= 1024) streams_step4_kernel<T, NS, 4><<<rows, 256, 0, stream>>>(a, h);
  else streams_step4_kernel<T, NS, 8><<<rows, 256, 0, stream>>>(a, h);
}

template <typename T>
void launch_streams(const StreamArgs& a, T* h, int rows, bool fours, hipStream_t stream) {
  if (!fours) {
    streams_step_kernel<T><<<rows, 256, 0, stream>>>(a, h);
    return;
  }
  switch (a.S) {
    case 1: launch_streams4<T, 1>(a, h, rows, stream); break;
    case 2: launch_streams4<T, 2>(a, h, rows, stream); break;
    case 3: launch_streams4<T, 3>(a, h, rows, stream); break;
    case 4: launch_streams4<T, 4>(a, h, rows, stream); break;
    default: launch_streams4<T, 0>(a, h, rows, stream); break;
  }
}

}  // namespace

// src: `streams` streams of [rows, width], src_stride floats apart (0: one stands for all).  y [pieces, rows, width] with
// mix [streams, streams] (from, to), out_w [streams] and dst [streams, rows, width]: the streams are written.  h (dtype
// h_dtype) with norm_w [width] (and read_w [streams], or null for the plain sum): what the next sublayer reads.
extern "C" int lq_streams_step(const float* src, long long src_stride, int streams, int rows, int width, const float* y,
                               int pieces, long long y_stride, const float* mix, const float* out_w, float* dst,
                               const float* read_w, const float* norm_w, float eps, void* h, int h_dtype,
                               hipStream_t stream) {
  LQ_REQUIRE(rows > 0 && width > 0 && streams >= 1 && streams <= MAX_STREAMS, "streams_step: %d streams of %d x %d (at most %d)",
             streams, rows, width, MAX_STREAMS);
  LQ_REQUIRE(src && (src_stride == 0 || src_stride >= (long long)rows * width), "streams_step: no streams, or streams that overlap");
  LQ_REQUIRE(y == nullptr || (pieces >= 1 && mix && out_w && dst), "streams_step: a result to write needs its weights and a place");
  LQ_REQUIRE(y != nullptr || h != nullptr, "streams_step: nothing to do");
  LQ_REQUIRE(h == nullptr || norm_w, "streams_step: what is read is normed");
  LQ_REQUIRE(h == nullptr || h_dtype == LQ_F32 || h_dtype == LQ_BF16, "streams_step: unknown dtype %d", h_dtype);
  StreamArgs a = {src, src_stride, dst, (long long)rows * width, y, pieces, y_stride, mix, out_w, read_w, norm_w, eps, streams, width};
  const bool fours = width % 4 == 0 && width <= 8192 && (uintptr_t)src % 16 == 0 && src_stride % 4 == 0 && y_stride % 4 == 0 &&
                     (uintptr_t)dst % 16 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)norm_w % 16 == 0 && (uintptr_t)h % 16 == 0;
  if (h_dtype == LQ_BF16) launch_streams<bf16_t>(a, (bf16_t*)h, rows, fours, stream);
  else launch_streams<float>(a, (float*)h, rows, fours, stream);
  LQ_CHECK_LAUNCH("streams_step");
  return 0;
}

extern "C" int lq_softcap(float* x, float cap, float factor, long long n, hipStream_t stream) {
  LQ_REQUIRE(x && n > 0 && cap > 0.f, "softcap: %lld entries under a cap of %g", n, (double)cap);
  softcap_kernel<<<(unsigned)((n + 255) / 256), 256, 0, stream>>>(x, cap, factor, n);
  LQ_CHECK_LAUNCH("softcap");
  return 0;
}
