// Several residual streams side by side (hyper-connections), and norms over a whole row.
//
//   stream_mix_norm   per token, the streams x_1 .. x_S (float32): every new stream takes a share of every old one and
//                     of the sublayer's output y that waits to be added,
//                         x'_t = sum_s mix[s, t] x_s + out[t] y,      y = the sum of up to four terms (and a bias),
//                     then what the next sublayer reads, u = sum_t read[t] x'_t, and a norm of u (a layer norm with
//                     weight and bias, or an RMS norm) in one pass over the streams. Every part may be absent: without
//                     mix nothing is mixed (x'_t = x_t, plus y where there are terms), without read u is the plain sum,
//                     without a weight u itself comes out. With an index per output row it works on chosen rows only
//                     (embedding rows by token, the rows that want logits). Rows that start the streams are one row
//                     [n] that all streams share (a stream stride of 0).
//
// Everything is float32; the result is rounded once.
#include "common.h"

#define HS_MAX_TERMS 4
#define HS_MAX_STREAMS 32

struct StreamArgs {
  const void* in; int in_dtype; int64_t row_stride, stream_stride;
  const int32_t* rows; int64_t in_rows;
  const void* term[HS_MAX_TERMS]; int dtype[HS_MAX_TERMS]; int parts[HS_MAX_TERMS]; int64_t part_stride[HS_MAX_TERMS]; int count;
  const float* y_bias;                                           // [n] or null: joins the sum of the terms
  const float* mix; const float* out_w; const float* read;      // [S, S] (from, to), [S], [S]
  float* streams_out;                                            // [T, S, n] or null
  const float* w; const float* b; int center; float eps;
  void* y; int S, n;
};

// W neighbours of a row as float32.
template <int W>
__device__ __forceinline__ void load_row(const void* p, int dtype, int64_t at, float (&v)[W]) {
  if (dtype == ME_F32) {
    if constexpr (W == 4) {
      const float4 t = *reinterpret_cast<const float4*>((const float*)p + at);
      v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
    } else v[0] = ((const float*)p)[at];
  } else {
    if constexpr (W == 4) {
      const bf16x4 t = *reinterpret_cast<const bf16x4*>((const bf16_t*)p + at);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = static_cast<float>(t[e]);
    } else v[0] = static_cast<float>(((const bf16_t*)p)[at]);
  }
}

template <int W>
__device__ __forceinline__ void store_row(float* p, const float (&v)[W]) {
  if constexpr (W == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else p[0] = v[0];
}
template <int W>
__device__ __forceinline__ void store_row(bf16_t* p, const float (&v)[W]) {
  if constexpr (W == 4) {
    bf16x4 t;
#pragma unroll
    for (int e = 0; e < 4; ++e) t[e] = static_cast<bf16_t>(v[e]);
    *reinterpret_cast<bf16x4*>(p) = t;
  } else p[0] = static_cast<bf16_t>(v[0]);
}

// One workgroup per output row; u stays in LDS between the sums and the norm. SC: the number of streams, known to the
// compiler (their values then stay in registers); 0: up to HS_MAX_STREAMS, asked for at run time. W: 4 neighbours at a
// time, or 1.
template <typename TY, int SC, int W>
__global__ void __launch_bounds__(1024) stream_mix_norm_kernel(StreamArgs a) {
  __shared__ float scratch[16];
  extern __shared__ __align__(16) float row[];
  constexpr int SM = SC > 0 ? SC : HS_MAX_STREAMS;
  const int S = SC > 0 ? SC : a.S;
  const int64_t r = blockIdx.x;
  int64_t src = r;
  if (a.rows) {
    src = a.rows[r];
    if (src < 0 || src >= a.in_rows) src = 0;           // the host bounds the indices; never read outside the rows
  }
  const int n = a.n;
  float total = 0.f;
  for (int i = threadIdx.x * W; i < n; i += blockDim.x * W) {
    float y[W];
#pragma unroll
    for (int e = 0; e < W; ++e) y[e] = 0.f;
    if (a.y_bias) load_row<W>(a.y_bias, ME_F32, i, y);
#pragma unroll
    for (int k = 0; k < HS_MAX_TERMS; ++k)
      if (k < a.count) {
        float v[W];
#pragma unroll
        for (int e = 0; e < W; ++e) v[e] = 0.f;
        for (int p = 0; p < a.parts[k]; ++p) {
          float x[W];
          load_row<W>(a.term[k], a.dtype[k], p * a.part_stride[k] + src * n + i, x);
#pragma unroll
          for (int e = 0; e < W; ++e) v[e] += x[e];
        }
#pragma unroll
        for (int e = 0; e < W; ++e) y[e] += v[e];
      }
    float old[SM][W], u[W];
#pragma unroll
    for (int e = 0; e < W; ++e) u[e] = 0.f;
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (s < S) load_row<W>(a.in, a.in_dtype, src * a.row_stride + s * a.stream_stride + i, old[s]);
#pragma unroll
    for (int t = 0; t < SM; ++t)
      if (t < S) {
        float x[W];
        if (a.mix) {
          const float ow = a.out_w[t];
#pragma unroll
          for (int e = 0; e < W; ++e) x[e] = ow * y[e];
#pragma unroll
          for (int s = 0; s < SM; ++s)
            if (s < S) {
              const float m = a.mix[s * S + t];
#pragma unroll
              for (int e = 0; e < W; ++e) x[e] = fmaf(m, old[s][e], x[e]);
            }
        } else {
#pragma unroll
          for (int e = 0; e < W; ++e) x[e] = old[t][e] + y[e];
        }
        if (a.streams_out) store_row<W>(a.streams_out + (r * S + t) * n + i, x);
        const float rd = a.read ? a.read[t] : 1.0f;
#pragma unroll
        for (int e = 0; e < W; ++e) u[e] = fmaf(rd, x[e], u[e]);
      }
    if (a.w == nullptr) {
      if (a.y) store_row<W>((TY*)a.y + r * n + i, u);
    } else {
#pragma unroll
      for (int e = 0; e < W; ++e) { row[i + e] = u[e]; total += u[e]; }
    }
  }
  if (a.w == nullptr) return;
  const float mean = a.center ? block_sum(total, scratch) / (float)n : 0.f;
  float ss = 0.f;
  for (int i = threadIdx.x * W; i < n; i += blockDim.x * W)
#pragma unroll
    for (int e = 0; e < W; ++e) { const float d = row[i + e] - mean; ss += d * d; }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)n + a.eps);
  for (int i = threadIdx.x * W; i < n; i += blockDim.x * W) {
    float v[W];
#pragma unroll
    for (int e = 0; e < W; ++e) {
      v[e] = (row[i + e] - mean) * inv * a.w[i + e];
      if (a.b) v[e] += a.b[i + e];
    }
    store_row<W>((TY*)a.y + r * n + i, v);
  }
}

template <typename TY, int W>
static void launch_stream_mix(const StreamArgs& a, int64_t R, int threads, hipStream_t stream) {
  const size_t lds = a.w ? (size_t)a.n * sizeof(float) : 0;
#define HS(SC) stream_mix_norm_kernel<TY, SC, W><<<dim3((unsigned)R), dim3(threads), lds, stream>>>(a)
  switch (a.S) {
    case 1: HS(1); break;
    case 2: HS(2); break;
    case 3: HS(3); break;
    case 4: HS(4); break;
    case 5: HS(5); break;
    case 6: HS(6); break;
    case 8: HS(8); break;
    default: HS(0); break;
  }
#undef HS
}

// in: rows [in_rows, ...] with `row_stride` elements from row to row and `stream_stride` from stream to stream (0: all
// streams share the row). rows: int32 [R] or null (R = in_rows then, row by row). terms: `count` entries [parts, in_rows, n].
extern "C" int me_stream_mix_norm(const void* in, int in_dtype, int64_t row_stride, int64_t stream_stride, const int32_t* rows,
                                  int64_t in_rows, int count, const void* const* term, const int* term_dtype, const int* term_parts,
                                  const int64_t* term_stride, const float* y_bias, const float* mix, const float* out_w, const float* read,
                                  float* streams_out, const float* w, const float* b, int center, float eps, void* y, int out_dtype,
                                  int64_t R, int S, int n, hipStream_t stream) {
  if (R == 0) return 0;
  ME_CHECK(n >= 1 && n <= 15360, "stream_mix_norm: width %d outside 1..15360", n);
  ME_CHECK(S >= 1 && S <= HS_MAX_STREAMS, "stream_mix_norm: %d streams outside 1..%d", S, HS_MAX_STREAMS);
  ME_CHECK(count >= 0 && count <= HS_MAX_TERMS, "stream_mix_norm: up to %d terms", HS_MAX_TERMS);
  ME_CHECK((mix == nullptr) == (out_w == nullptr), "stream_mix_norm: a mix comes with the output's weights");
  ME_CHECK(R < (1ll << 31) && in_rows >= 1 && (rows != nullptr || R <= in_rows), "stream_mix_norm: too many rows");
  ME_CHECK(y != nullptr || w == nullptr, "stream_mix_norm: a norm needs a place for its result");
  StreamArgs a;
  a.in = in; a.in_dtype = in_dtype; a.row_stride = row_stride; a.stream_stride = stream_stride; a.rows = rows; a.in_rows = in_rows;
  a.count = count; a.y_bias = y_bias; a.mix = mix; a.out_w = out_w; a.read = read; a.streams_out = streams_out; a.w = w; a.b = b; a.center = center;
  a.eps = eps; a.y = y; a.S = S; a.n = n;
  uintptr_t bits = reinterpret_cast<uintptr_t>(in) | reinterpret_cast<uintptr_t>(streams_out) | reinterpret_cast<uintptr_t>(y) |
                   reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(b) | reinterpret_cast<uintptr_t>(y_bias);
  bool vec = n % 4 == 0 && row_stride % 4 == 0 && stream_stride % 4 == 0;
  for (int k = 0; k < HS_MAX_TERMS; ++k) {
    const bool on = k < count;
    a.term[k] = on ? term[k] : nullptr; a.dtype[k] = on ? term_dtype[k] : ME_F32; a.parts[k] = on ? term_parts[k] : 0;
    a.part_stride[k] = on ? term_stride[k] : 0;
    if (!on) continue;
    ME_CHECK(a.parts[k] >= 1 && a.parts[k] <= 64 && (a.parts[k] == 1 || a.dtype[k] == ME_F32), "stream_mix_norm: 1 to 64 float32 partial sums");
    bits |= reinterpret_cast<uintptr_t>(a.term[k]);
    vec = vec && a.part_stride[k] % 4 == 0;
  }
  vec = vec && bits % 16 == 0;
  // few rows: a row's threads are all the launch has, so as many as its groups fill; many rows: 256
  const int per = vec ? 4 : 1;
  int threads = R >= 512 ? 256 : 1024;
  while (threads > 64 && threads * per / 2 >= n) threads >>= 1;
  if (out_dtype == ME_F32) { if (vec) launch_stream_mix<float, 4>(a, R, threads, stream); else launch_stream_mix<float, 1>(a, R, threads, stream); }
  else { if (vec) launch_stream_mix<bf16_t, 4>(a, R, threads, stream); else launch_stream_mix<bf16_t, 1>(a, R, threads, stream); }
  ME_LAUNCH_CHECK();
  return 0;
}
