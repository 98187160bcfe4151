// Row kernel of a layer with several residual streams (hyper-connections). A sublayer reads the norm of a weighted sum of
// the streams, and its result y changes all of them at once:
//
//   X_t <- sum_s mix[s, t] X_s + out[t] y
//
// One kernel a sublayer does what is pending from the sublayer before (its y, with that sublayer's mix and out) and what
// the next one needs: u = sum_t in[t] X_t of the new streams, and u / sqrt(mean u^2 + eps) * w in the activations' type.
// Streams, sums and the norm are float. At the model's start all streams are the embedding: they are read from one row
// (base) until the first y has made them differ.
#include "common.h"
#include "reinfer_hip.h"

namespace {

struct HyperArgs {
  float* streams;              // [T][n][h]
  const float* base;           // [T][h] where every stream is still this row, or null
  const void* y;               // [T][h], or null: nothing pending
  const float* mix;            // [n][n], from and to
  const float* w_out;          // [n]
  const float* w_in;           // [n], or null: ones
  const float* weight;         // [h] of the norm, or null: u as it is
  float eps;
  const int* rows;             // which rows, into a compact result; nothing is stored into the streams then; or null
  int h, n, store;
  void* out;                   // [rows][h], or null
};

// Rows whose width is a multiple of 4: a thread holds CH runs of four neighbouring elements of every stream in registers,
// everything it reads is asked for in one trip to memory.
template <typename TY, typename TO, int N, int CH>
__global__ void __launch_bounds__(CH == 1 ? 1024 : 512) hyper_step_kernel(HyperArgs p) {
  __shared__ float red[17];
  const int h = p.h;
  const size_t t = p.rows ? (size_t)p.rows[blockIdx.x] : (size_t)blockIdx.x;
  float* X = p.streams + t * N * h;
  f32x4_t x[CH][N], y[CH], w[CH];
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int e = (threadIdx.x + c * blockDim.x) * 4;
    y[c] = w[c] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < N; ++s) x[c][s] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    if (e >= h) continue;
    if (p.base) {
      x[c][0] = *(const f32x4_t*)(p.base + t * h + e);
    } else {
#pragma unroll
      for (int s = 0; s < N; ++s) x[c][s] = *(const f32x4_t*)(X + (size_t)s * h + e);
    }
    if (p.y) {
      if constexpr (sizeof(TY) == 4) {
        y[c] = *(const f32x4_t*)((const float*)p.y + t * h + e);
      } else {
        const bf16x4_t b = *(const bf16x4_t*)((const bf16_t*)p.y + t * h + e);
        y[c] = (f32x4_t){(float)b[0], (float)b[1], (float)b[2], (float)b[3]};
      }
    }
    if (p.weight) w[c] = *(const f32x4_t*)(p.weight + e);
  }
  float mix[N][N], wo[N], wi[N];
#pragma unroll
  for (int s = 0; s < N; ++s) {
    wo[s] = p.y ? p.w_out[s] : 0.f;
    wi[s] = p.w_in ? p.w_in[s] : 1.f;
#pragma unroll
    for (int u = 0; u < N; ++u) mix[s][u] = p.y ? p.mix[s * N + u] : (s == u ? 1.f : 0.f);
  }
  f32x4_t u[CH];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int e = (threadIdx.x + c * blockDim.x) * 4;
    if (p.base) {
#pragma unroll
      for (int s = 1; s < N; ++s) x[c][s] = x[c][0];
    }
    u[c] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int to = 0; to < N; ++to) {
      f32x4_t z = x[c][to];
      if (p.y) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float v = 0.f;
#pragma unroll
          for (int s = 0; s < N; ++s) v += mix[s][to] * x[c][s][i];
          z[i] = v + wo[to] * y[c][i];
        }
      }
      if (p.store && e < h) *(f32x4_t*)(X + (size_t)to * h + e) = z;
#pragma unroll
      for (int i = 0; i < 4; ++i) u[c][i] += wi[to] * z[i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) ss += u[c][i] * u[c][i];
  }
  if (!p.out) return;
  float rstd = 1.f;
  if (p.weight) rstd = 1.f / sqrtf(block_sum(ss, red) / (float)h + p.eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int e = (threadIdx.x + c * blockDim.x) * 4;
    if (e >= h) continue;
    float o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = p.weight ? u[c][i] * rstd * w[c][i] : u[c][i];
    const size_t at = (size_t)blockIdx.x * h + e;
    if constexpr (sizeof(TO) == 4) *(f32x4_t*)((float*)p.out + at) = (f32x4_t){o[0], o[1], o[2], o[3]};
    else *(bf16x4_t*)((bf16_t*)p.out + at) = (bf16x4_t){(bf16_t)o[0], (bf16_t)o[1], (bf16_t)o[2], (bf16_t)o[3]};
  }
}

// Any width and any number of streams up to HYPER_MAX: element by element, the row's u in a buffer of LDS or, where that
// is too small, formed again.
#define HYPER_MAX 64
#define HYPER_ROW 8192
template <typename TY, typename TO>
__global__ void hyper_step_any_kernel(HyperArgs p) {
  __shared__ float red[17];
  __shared__ float row_u[HYPER_ROW];
  const int h = p.h, n = p.n;
  const size_t t = p.rows ? (size_t)p.rows[blockIdx.x] : (size_t)blockIdx.x;
  float* X = p.streams + t * n * h;
  const TY* y = (const TY*)p.y;
  const bool keep = h <= HYPER_ROW;
  auto element = [&](int e, bool store) -> float {       // u of one element; the new streams where asked
    float old[HYPER_MAX];
    float yv = y ? to_f32(y[t * h + e]) : 0.f, u = 0.f;
    for (int s = 0; s < n; ++s) old[s] = p.base ? p.base[t * h + e] : X[(size_t)s * h + e];
    for (int to = 0; to < n; ++to) {
      float z = old[to];
      if (y) {
        float v = 0.f;
        for (int s = 0; s < n; ++s) v += p.mix[s * n + to] * old[s];
        z = v + p.w_out[to] * yv;
      }
      if (store) X[(size_t)to * h + e] = z;
      u += (p.w_in ? p.w_in[to] : 1.f) * z;
    }
    return u;
  };
  float ss = 0.f;
  for (int e = threadIdx.x; e < h; e += blockDim.x) {
    const float u = element(e, p.store && keep);
    if (keep) row_u[e] = u;                              // a thread reads back what it wrote itself
    ss += u * u;
  }
  float rstd = 1.f;
  if (p.weight) rstd = 1.f / sqrtf(block_sum(ss, red) / (float)h + p.eps);
  for (int e = threadIdx.x; e < h; e += blockDim.x) {
    const float u = keep ? row_u[e] : element(e, p.store);
    if (p.out) ((TO*)p.out)[(size_t)blockIdx.x * h + e] = from_f32<TO>(p.weight ? u * rstd * p.weight[e] : u);
  }
}

template <typename TY, typename TO, int N>
bool hyper_vec(const HyperArgs& a, int n_rows, hipStream_t stream) {
  // few rows: as many threads a row as there are; many rows: fewer threads, each with more in flight
  const int quads = a.h / 4;
  int ch = n_rows < 512 && quads <= 1024 ? 1 : quads <= 256 ? 1 : quads <= 512 ? 2 : 4;
  const int threads = ((quads + ch - 1) / ch + RA_WAVE - 1) / RA_WAVE * RA_WAVE;
  if (threads > (ch == 1 ? 1024 : 512)) return false;      // wider rows: the general form
  if (ch == 1) hyper_step_kernel<TY, TO, N, 1><<<n_rows, threads, 0, stream>>>(a);
  else if (ch == 2) hyper_step_kernel<TY, TO, N, 2><<<n_rows, threads, 0, stream>>>(a);
  else hyper_step_kernel<TY, TO, N, 4><<<n_rows, threads, 0, stream>>>(a);
  return true;
}

template <typename TY, typename TO>
void hyper_dispatch(const HyperArgs& a, bool vec, int n_rows, hipStream_t stream) {
  bool done = false;
  if (vec) {
    switch (a.n) {
      case 1: done = hyper_vec<TY, TO, 1>(a, n_rows, stream); break;
      case 2: done = hyper_vec<TY, TO, 2>(a, n_rows, stream); break;
      case 3: done = hyper_vec<TY, TO, 3>(a, n_rows, stream); break;
      case 4: done = hyper_vec<TY, TO, 4>(a, n_rows, stream); break;
      case 5: done = hyper_vec<TY, TO, 5>(a, n_rows, stream); break;
      case 6: done = hyper_vec<TY, TO, 6>(a, n_rows, stream); break;
      case 8: done = hyper_vec<TY, TO, 8>(a, n_rows, stream); break;
      default: break;
    }
  }
  if (!done) hyper_step_any_kernel<TY, TO><<<n_rows, a.h >= 1024 ? 1024 : 256, 0, stream>>>(a);
}

}  // namespace

extern "C" int ra_hyper_step(float* streams, const float* base, const void* y, int y_dtype, const float* mix, const float* w_out,
                             const float* w_in, const float* weight, float eps, const int* rows, int n_rows, int n_streams,
                             int hidden, int store, void* out, int out_dtype, hipStream_t stream) {
  RA_CHECK(n_rows > 0 && hidden > 0, "hyper_step: %d rows of %d", n_rows, hidden);
  RA_CHECK(n_streams >= 1 && n_streams <= HYPER_MAX, "hyper_step: %d streams (1 to %d)", n_streams, HYPER_MAX);
  RA_CHECK(streams != nullptr && (out != nullptr || store), "hyper_step: nothing to compute");
  RA_CHECK(y == nullptr || (mix && w_out), "hyper_step: a result enters the streams by its mix and its factors");
  RA_CHECK(!(rows && store), "hyper_step: chosen rows are read only");
  HyperArgs a = {};
  a.streams = streams; a.base = base; a.y = y; a.mix = mix; a.w_out = w_out; a.w_in = w_in; a.weight = weight; a.eps = eps;
  a.rows = rows; a.h = hidden; a.n = n_streams; a.store = store; a.out = out;
  const bool vec = hidden % 4 == 0 && ((uintptr_t)streams % 16) == 0 && ((uintptr_t)base % 16) == 0 && ((uintptr_t)y % 16) == 0 &&
                   ((uintptr_t)weight % 16) == 0 && ((uintptr_t)out % 16) == 0;
#define RA_HS(TY, TO) hyper_dispatch<TY, TO>(a, vec, n_rows, stream)
  if (y_dtype == RA_F32 && out_dtype == RA_F32) RA_HS(float, float);
  else if (y_dtype == RA_F32 && out_dtype == RA_BF16) RA_HS(float, bf16_t);
  else if (y_dtype == RA_BF16 && out_dtype == RA_BF16) RA_HS(bf16_t, bf16_t);
  else if (y_dtype == RA_BF16 && out_dtype == RA_F32) RA_HS(bf16_t, float);
  else return ra_fail("hyper_step: unknown dtype tags %d, %d", y_dtype, out_dtype);
#undef RA_HS
  RA_LAUNCH_CHECK("hyper_step");
  return 0;
}
