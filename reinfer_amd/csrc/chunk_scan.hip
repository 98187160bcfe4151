// Linear attention with a decay, a prompt's portion in chunks of 16 tokens on the float matrix cores.
//
//   S_t = A_t S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t          per head, S [dk, dv] float, from and into the request's slot
//
// with A_t one factor a head (mode FIXED: a memory that fades by a constant, retention) or one a key channel and token
// (mode CHANNEL: gated linear attention). Token by token this is a chain of as many steps as there are tokens; a chunk
// of C = 16 tokens is a handful of 16 x 16 products instead. With B_i the product of the factors from the chunk's first
// token to its i-th, S the state before the chunk:
//
//   o_i = (B_i q_i)^T S + sum_(j <= i) (q_i . (B_i / B_j) k_j) v_j
//   S'  = B_C S + sum_j ((B_C / B_j) k_j) v_j^T
//
// Everything is float: the products are v_mfma_f32_16x16x4_f32, the state stays in the accumulators of the waves from
// the portion's first chunk to its last. A workgroup is one (request, head, 16 columns of v); its four waves split dk.
// The accumulator of a 16 x 16 product (row 4 g + i, column r in lane 16 g + r, register i) is at the same time the
// operand of a product over those rows, if step i of four takes rows {i, 4 + i, 8 + i, 12 + i}: so S is used where it
// lies, and so are the scores (computed transposed, K Q^T). The waves' parts of o meet in LDS.
//
// Factors. FIXED: powers of the head's factor, none above 1: on the scores' accumulator, on the rows of Q S, on v's
// operand. CHANNEL: log2 of B is prepared beforehand (chunk_decay_kernel); B_i and B_C / B_j are at most 1; the scores
// are the product of B_i q_i with k_j / B_j where no channel of the wave falls below 2^-60 inside the chunk, else they
// are summed pair by pair with B_i / B_j, which never overflows.
//
// The state's layout in the slot is the token-by-token kernel's (scan_geom.h): steps may change from one to the other.
#include "common.h"
#include "reinfer_hip.h"
#include "scan_geom.h"

namespace {

#define CS_C 16                 // tokens of a chunk
#define CS_VP 20                // floats between rows of v, and of the waves' parts of o, in LDS
#define CS_LIMIT 60.f           // log2 of the smallest factor that the product form of the scores takes

enum { CS_FIXED = 0, CS_CHANNEL = 1 };

struct ChunkArgs {
  const void* q; const void* k; const void* v;      // column 0 of each in row 0; rows ld elements apart
  int ld;
  float q_scale, k_scale;
  int silu;                                          // q, k and v pass silu
  const float2* turn; int rot_dims;                  // (cos, sin) [T][rot_dims / 2] of q's and k's first elements, or none
  const float* head_decay;                           // FIXED: one factor a head
  const float* cum;                                  // CHANNEL: log2 B [T][H dk], from the start of each chunk on
  float* state; long slot_stride;
  const int* cu_tokens; const int* state_slots; const int* fresh;
  int n_seqs, H, dk, dv, waves_per_head, wave_floats, R, NPL, CPW;
  int vec;                                           // rows of q and k in whole 16-byte pieces of 8 elements
  float* out;                                        // [T][H dv]
};

// Eight elements as they lie in memory: nothing is computed on them until they are needed.
template <typename TA> struct Run8;
template <> struct Run8<bf16_t> {
  bf16x8_t a;
  __device__ __forceinline__ void load(const bf16_t* p) { a = *(const bf16x8_t*)p; }
  __device__ __forceinline__ void zero() { a = (bf16x8_t){0, 0, 0, 0, 0, 0, 0, 0}; }
  __device__ __forceinline__ float at(int i) const { return (float)a[i]; }
};
template <> struct Run8<float> {
  f32x4_t a, b;
  __device__ __forceinline__ void load(const float* p) { a = *(const f32x4_t*)p; b = *(const f32x4_t*)(p + 4); }
  __device__ __forceinline__ void zero() { a = b = (f32x4_t){0.f, 0.f, 0.f, 0.f}; }
  __device__ __forceinline__ float at(int i) const { return i < 4 ? a[i & 3] : b[i & 3]; }
};

__device__ __forceinline__ float silu_fast(float x) { return __fdividef(x, 1.f + __expf(-x)); }
__device__ __forceinline__ float power(float d, int n) {       // d^n, n in 0..16
  float r = 1.f;
#pragma unroll
  for (int b = 0; b < 5; ++b) {
    if ((n >> b) & 1) r *= d;
    d *= d;
  }
  return r;
}

// NT: 16-row tiles of S a wave holds (a head's dk padded to 64 NT)
template <typename TA, int NT, int MODE>
__global__ void __launch_bounds__(256) chunk_scan_kernel(ChunkArgs p) {
  constexpr bool CHANNEL = MODE == CS_CHANNEL;
  constexpr int DKP = 64 * NT, PITCH = DKP + 4;
  constexpr int SEGS = DKP / 8;                      // runs of 8 elements of a row
  constexpr int J = (CS_C * SEGS + 255) / 256;       // runs a thread stages
  constexpr int ROWS = CS_C * PITCH;
  constexpr int BUF = ROWS * (CHANNEL ? 3 : 2) + CS_C * CS_VP;
  extern __shared__ __attribute__((aligned(16))) float lds[];      // two buffers [q | k | log2 B | v], two of the waves' parts
  float* red = lds + 2 * BUF;

  const int tid = threadIdx.x, lane = tid & (RA_WAVE - 1), wave = tid / RA_WAVE;
  const int r = lane & 15, g = lane >> 4;
  // the column groups of one (request, head) read the same q and k: they are given to one XCD
  const int CG = (p.dv + 15) / 16;
  const int rest = blockIdx.x / RA_XCDS;
  const int unit = (rest / CG) * RA_XCDS + blockIdx.x % RA_XCDS, cg = rest % CG;
  if (unit >= p.n_seqs * p.H) return;
  const int seq = unit / p.H, head = unit % p.H;
  const int first = p.cu_tokens[seq], last = p.cu_tokens[seq + 1];
  const int slot = p.state_slots[seq];
  const size_t ow = (size_t)p.H * p.dv;
  const int tok = tid / 16, vc = tid % 16;           // the (token, column) this thread stages of v and writes of o
  const int vcol = cg * 16 + vc;
  const bool v_ok = vcol < p.dv;
  if (slot < 0) {                                    // a padding row: no state, a defined result
    for (int t = first + tok; t < last; t += 16)
      if (v_ok) p.out[(size_t)t * ow + (size_t)head * p.dv + vcol] = 0.f;
    return;
  }
  if (first >= last) return;

  const int dk = p.dk;
  const TA* qg = (const TA*)p.q + (size_t)head * dk;
  const TA* kg = (const TA*)p.k + (size_t)head * dk;
  const TA* vg = (const TA*)p.v + (size_t)head * p.dv + vcol;
  const int half = p.rot_dims >> 1;

  // ---- what a thread stages: runs of 8 elements, the same places in every chunk
  Run8<TA> fq[J], fk[J], pq[J], pk[J];
  float2 cs[J][8];
  float fb[CHANNEL ? J : 1][8];
  TA fv = (TA)0.f;
  const bool turn_vec = p.vec && p.rot_dims > 0 && half % 8 == 0;      // pairs lie whole runs apart
  auto fetch = [&](int t0) {                         // loads only
    const int n = min(CS_C, last - t0);
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const int idx = tid + j * 256, t = idx / SEGS, e = (idx % SEGS) * 8;
      fq[j].zero();
      fk[j].zero();
      if (p.vec && t < n && e < dk) {
        const size_t at = (size_t)(t0 + t) * p.ld + e;
        fq[j].load(qg + at);
        fk[j].load(kg + at);
        if (turn_vec && e < p.rot_dims) {
          const int o = e < half ? half : -half;
          pq[j].load(qg + at + o);
          pk[j].load(kg + at + o);
          const float2* tp = p.turn + (size_t)(t0 + t) * half + (e < half ? e : e - half);
#pragma unroll
          for (int i = 0; i < 8; ++i) cs[j][i] = tp[i];
        }
      }
      if (CHANNEL) {
        const bool in = t < n && e < dk;
        const float* bp = p.cum + (size_t)(t0 + t) * p.H * dk + (size_t)head * dk + e;
        if (p.vec && in) {
          Vec8<float>::load(bp, fb[j]);
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i) fb[j][i] = (in && e + i < dk) ? bp[i] : 0.f;
        }
      }
    }
    fv = (v_ok && tok < n) ? vg[(size_t)(t0 + tok) * p.ld] : (TA)0.f;
  };
  auto stage = [&](int t0, float* buf) {             // registers -> LDS, as the products want them
    const int n = min(CS_C, last - t0);
#pragma unroll
    for (int j = 0; j < J; ++j) {
      const int idx = tid + j * 256, t = idx / SEGS, e = (idx % SEGS) * 8;
      if (t >= CS_C) continue;
      float q8[8], k8[8];
      if (p.vec) {
#pragma unroll
        for (int i = 0; i < 8; ++i) { q8[i] = fq[j].at(i); k8[i] = fk[j].at(i); }
        if (p.silu) {
#pragma unroll
          for (int i = 0; i < 8; ++i) { q8[i] = silu_fast(q8[i]); k8[i] = silu_fast(k8[i]); }
        }
        if (turn_vec && t < n && e < p.rot_dims) {
          const float sign = e < half ? -1.f : 1.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const float sn = sign * cs[j][i].y;
            q8[i] = q8[i] * cs[j][i].x + pq[j].at(i) * sn;
            k8[i] = k8[i] * cs[j][i].x + pk[j].at(i) * sn;
          }
        }
      } else {                                       // element by element, straight from memory
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          q8[i] = k8[i] = 0.f;
          if (t < n && e + i < dk) {
            const size_t at = (size_t)(t0 + t) * p.ld + e + i;
            q8[i] = to_f32(qg[at]);
            k8[i] = to_f32(kg[at]);
            if (p.silu) { q8[i] = silu_fast(q8[i]); k8[i] = silu_fast(k8[i]); }
          }
        }
      }
      if (!turn_vec && p.rot_dims > 0 && t < n && e < p.rot_dims) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int x = e + i;
          if (x < p.rot_dims) {
            const bool lower = x < half;
            const size_t at = (size_t)(t0 + t) * p.ld + x + (lower ? half : -half);
            const float2 c = p.turn[(size_t)(t0 + t) * half + (lower ? x : x - half)];
            const float sn = lower ? -c.y : c.y;
            q8[i] = q8[i] * c.x + to_f32(qg[at]) * sn;
            k8[i] = k8[i] * c.x + to_f32(kg[at]) * sn;
          }
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) { q8[i] *= p.q_scale; k8[i] *= p.k_scale; }
      Vec8<float>::store(buf + t * PITCH + e, q8);
      Vec8<float>::store(buf + ROWS + t * PITCH + e, k8);
      if (CHANNEL) Vec8<float>::store(buf + 2 * ROWS + t * PITCH + e, fb[j]);
    }
    float v = to_f32(fv);
    if (p.silu) v = silu_fast(v);
    buf[ROWS * (CHANNEL ? 3 : 2) + tok * CS_VP + vc] = v;
  };

  // ---- the state: tile nt of the wave is rows base + 16 nt + 4 g + i, column r of the group
  const int base = wave * 16 * NT;
  const int col = cg * 16 + r;
  float* st = p.state + (size_t)slot * p.slot_stride +
              ((size_t)head * p.waves_per_head + (col < p.dv ? col : 0) / p.CPW) * p.wave_floats + (size_t)((col < p.dv ? col : 0) % p.CPW) * p.R;
  const int kept_rows = p.R * p.NPL;                 // elements of a column that the slot holds
  f32x4_t S[NT];
  const bool from_zero = p.fresh[seq] != 0;
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = base + 16 * nt + 4 * g + i;
      S[nt][i] = (!from_zero && col < p.dv && e < dk) ? st[(size_t)(e % p.NPL) * RA_WAVE + e / p.NPL] : 0.f;
    }

  // ---- FIXED: the head's powers at this lane's places
  const float d = CHANNEL ? 1.f : p.head_decay[head];
  float f_score[4], f_out[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int j = 4 * g + i;
    f_score[i] = (r >= j) ? (CHANNEL ? 1.f : power(d, r - j)) : 0.f;   // score of query r on key j
    f_out[i] = CHANNEL ? 1.f : power(d, j + 1);                        // row j of Q S
  }

  fetch(first);
  stage(first, lds);
  __syncthreads();
  int which = 0;
  for (int t0 = first; t0 < last; t0 += CS_C) {
    const int n = min(CS_C, last - t0);
    const bool more = t0 + CS_C < last;
    if (more) fetch(t0 + CS_C);
    const float* Q = lds + which * BUF;
    const float* K = Q + ROWS;
    const float* B = Q + 2 * ROWS;
    const float* V = Q + ROWS * (CHANNEL ? 3 : 2);
    f32x4_t o = {0.f, 0.f, 0.f, 0.f}, a = {0.f, 0.f, 0.f, 0.f};
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = V[(4 * g + i) * CS_VP + r];

    bool direct = false;                             // the scores pair by pair
    if (CHANNEL) {
      float low = 0.f;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const f32x4_t b = *(const f32x4_t*)(B + (n - 1) * PITCH + base + 16 * nt + 4 * g);
        low = fminf(low, fminf(fminf(b[0], b[1]), fminf(b[2], b[3])));
      }
      direct = __any(!(low >= -CS_LIMIT));
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int at = r * PITCH + base + 16 * nt + 4 * g;
      f32x4_t q = *(const f32x4_t*)(Q + at), k = *(const f32x4_t*)(K + at);
      if (CHANNEL) {
        const f32x4_t b = *(const f32x4_t*)(B + at);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          q[i] *= __builtin_amdgcn_exp2f(b[i]);
          if (!direct) k[i] *= __builtin_amdgcn_exp2f(-b[i]);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(q[i], S[nt][i], o, 0, 0, 0);
        if (!CHANNEL || !direct) a = __builtin_amdgcn_mfma_f32_16x16x4f32(k[i], q[i], a, 0, 0, 0);
      }
    }
    if (CHANNEL && direct) {                         // score of query r on keys 4 g + i, the wave's channels
      for (int c = base; c < base + 16 * NT; ++c) {
        const float bq = B[r * PITCH + c], qv = Q[r * PITCH + c];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int j = 4 * g + i;
          a[i] += qv * K[j * PITCH + c] * __builtin_amdgcn_exp2f(fminf(bq - B[j * PITCH + c], 0.f));
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      o[i] *= f_out[i];
      a[i] = (r >= 4 * g + i) ? a[i] * f_score[i] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], v[i], o, 0, 0, 0);

    // ---- the state moves on
    if (!CHANNEL) {
      const float dn = power(d, n);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] *= power(d, max(n - 1 - (4 * g + i), 0));     // rows past n are zeros
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
#pragma unroll
        for (int i = 0; i < 4; ++i) S[nt][i] *= dn;
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int c0 = base + 16 * nt;
      float bl = 0.f;
      if (CHANNEL) {
        const f32x4_t b = *(const f32x4_t*)(B + (n - 1) * PITCH + c0 + 4 * g);
#pragma unroll
        for (int i = 0; i < 4; ++i) S[nt][i] *= __builtin_amdgcn_exp2f(b[i]);
        bl = B[(n - 1) * PITCH + c0 + r];
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int at = (4 * g + i) * PITCH + c0 + r;
        float k = K[at];
        if (CHANNEL) k *= __builtin_amdgcn_exp2f(fminf(bl - B[at], 0.f));            // rows past n hold k = 0
        S[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, v[i], S[nt], 0, 0, 0);
      }
    }

    // ---- the waves' parts of o
    float* part = red + which * (4 * CS_C * CS_VP);
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave * CS_C * CS_VP + (4 * g + i) * CS_VP + r] = o[i];
    if (more) stage(t0 + CS_C, lds + (which ^ 1) * BUF);
    __syncthreads();
    if (tok < n && v_ok) {
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) s += part[w * CS_C * CS_VP + tok * CS_VP + vc];
      p.out[(size_t)(t0 + tok) * ow + (size_t)head * p.dv + vcol] = s;
    }
    which ^= 1;
  }
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = base + 16 * nt + 4 * g + i;
      if (col < p.dv && e < kept_rows) st[(size_t)(e % p.NPL) * RA_WAVE + e / p.NPL] = S[nt][i];
    }
}

// (cos, sin) of position * inv_freq[j] for every token and pair
__global__ void turn_table_kernel(const int* __restrict__ positions, const float* __restrict__ inv_freq, int half,
                                  float2* __restrict__ out, long n) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= n) return;
  float sn, cs;
  sincosf((float)positions[i / half] * inv_freq[i % half], &sn, &cs);
  out[i] = make_float2(cs, sn);
}

// z [T][C] (rows ldz apart) -> log2 of the products of sigmoid(z + bias)^inv_tau from each chunk's first token on; chunks
// of 16 tokens are counted from the start of the request's portion. One thread a (chunk, channel).
__global__ void chunk_decay_kernel(const float* __restrict__ z, int ldz, const float* __restrict__ bias, float inv_tau,
                                   const int* __restrict__ cu_tokens, int C, float* __restrict__ cum) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int seq = blockIdx.z;
  const int first = cu_tokens[seq] + blockIdx.y * CS_C, last = min(first + CS_C, cu_tokens[seq + 1]);
  if (c >= C || first >= last) return;
  const float b = bias[c], scale = inv_tau * 1.4426950408889634f;
  float x[CS_C];
#pragma unroll
  for (int i = 0; i < CS_C; ++i) x[i] = first + i < last ? z[(size_t)(first + i) * ldz + c] : 0.f;
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < CS_C; ++i)
    if (first + i < last) {
      sum += ra_logsigmoid(x[i] + b) * scale;
      cum[(size_t)(first + i) * C + c] = sum;
    }
}

template <typename TA, int NT, int MODE>
int chunk_launch(const ChunkArgs& a, hipStream_t stream) {
  constexpr int rows = CS_C * (64 * NT + 4);
  constexpr size_t bytes = (size_t)(2 * (rows * (MODE == CS_CHANNEL ? 3 : 2) + CS_C * CS_VP) + 2 * 4 * CS_C * CS_VP) * sizeof(float);
  if (bytes > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute((const void*)chunk_scan_kernel<TA, NT, MODE>,
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
    if (e != hipSuccess) return ra_fail("chunk_scan: the device does not give a workgroup %zu bytes of LDS", bytes);
  }
  const long units = ((long)a.n_seqs * a.H + RA_XCDS - 1) / RA_XCDS * RA_XCDS;
  const long grid = units * ((a.dv + 15) / 16);
  RA_CHECK(grid <= 0x7fffffffL, "chunk_scan: too many workgroups");
  chunk_scan_kernel<TA, NT, MODE><<<(unsigned)grid, 256, bytes, stream>>>(a);
  RA_LAUNCH_CHECK("chunk_scan");
  return 0;
}

template <typename TA, int MODE>
int chunk_pick(const ChunkArgs& a, hipStream_t stream) {
  const int rows = a.R * a.NPL;
  if (rows <= 64) return chunk_launch<TA, 1, MODE>(a, stream);
  if (rows <= 128) return chunk_launch<TA, 2, MODE>(a, stream);
  return chunk_launch<TA, 4, MODE>(a, stream);
}

int chunk_common(ChunkArgs& a, const char* what, int kind, const void* proj, int act_dtype, int ld, int q_off, int k_off,
                 int v_off, float* state, long slot_stride, int n_tokens) {
  RA_CHECK(a.n_seqs > 0 && n_tokens > 0 && a.H > 0, "%s: %d requests, %d tokens, %d heads", what, a.n_seqs, n_tokens, a.H);
  RA_CHECK(act_dtype == RA_F32 || act_dtype == RA_BF16, "%s: unknown dtype tag %d", what, act_dtype);
  ScanGeom g;
  RA_CHECK(scan_geom(kind, a.dk, a.dv, &g) && a.dk <= 256, "%s: heads of %d x %d (keys up to 256)", what, a.dk, a.dv);
  RA_CHECK(slot_stride >= (long)a.H * g.waves * g.wave_floats, "%s: a state slot of %ld floats, need %ld", what, slot_stride,
           (long)a.H * g.waves * g.wave_floats);
  const size_t es = act_dtype == RA_F32 ? 4 : 2;
  a.q = (const char*)proj + (size_t)q_off * es;
  a.k = (const char*)proj + (size_t)k_off * es;
  a.v = (const char*)proj + (size_t)v_off * es;
  a.ld = ld; a.state = state; a.slot_stride = slot_stride;
  a.waves_per_head = g.waves; a.wave_floats = g.wave_floats; a.R = g.R; a.NPL = g.NPL; a.CPW = g.CPW;
  a.vec = a.dk % 8 == 0 && ld % 8 == 0 && ((uintptr_t)a.q % 16) == 0 && ((uintptr_t)a.k % 16) == 0 && ((uintptr_t)a.cum % 16) == 0;
  return 0;
}

}  // namespace

// The recurrence of ra_decay_scan (silu) and ra_retention_scan in chunks, for steps with portions; the same state.
// turn: scratch of n_tokens * rot_dims floats where rot_dims > 0.
extern "C" int ra_decay_chunks(const void* proj, int act_dtype, int ld, int q_off, int k_off, int v_off, int silu,
                               const float* decays, const int* positions, const float* inv_freq, int rot_dims, float* turn,
                               float q_scale, float k_scale, float* state, long slot_stride, const int* cu_tokens,
                               const int* state_slots, const int* fresh, int n_seqs, int n_tokens, int heads, int key_dim,
                               int value_dim, float* out, hipStream_t stream) {
  RA_CHECK(decays != nullptr, "decay_chunks: one factor a head is needed");
  RA_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= key_dim && (rot_dims == 0 || (positions && inv_freq && turn && !silu)),
           "decay_chunks: %d turned elements of %d", rot_dims, key_dim);
  ChunkArgs a = {};
  a.n_seqs = n_seqs; a.H = heads; a.dk = key_dim; a.dv = value_dim;
  a.cu_tokens = cu_tokens; a.state_slots = state_slots; a.fresh = fresh; a.out = out;
  a.q_scale = q_scale; a.k_scale = k_scale; a.silu = silu; a.head_decay = decays; a.rot_dims = rot_dims;
  const int rc = chunk_common(a, "decay_chunks", 3, proj, act_dtype, ld, q_off, k_off, v_off, state, slot_stride, n_tokens);
  if (rc != 0) return rc;
  if (rot_dims > 0) {
    const long n = (long)n_tokens * (rot_dims / 2);
    turn_table_kernel<<<(unsigned)((n + 255) / 256), 256, 0, stream>>>(positions, inv_freq, rot_dims / 2, (float2*)turn, n);
    RA_LAUNCH_CHECK("turn_table");
    a.turn = (const float2*)turn;
  }
  return act_dtype == RA_F32 ? chunk_pick<float, CS_FIXED>(a, stream) : chunk_pick<bf16_t, CS_FIXED>(a, stream);
}

// The recurrence of ra_gla_scan in chunks. cum: scratch of n_tokens * heads * key_dim floats, 16-byte aligned.
extern "C" int ra_gla_chunks(const void* proj, int act_dtype, int ld, int q_off, int k_off, int v_off, const float* z, int ldz,
                             const float* bias, float tau, float* cum, float q_scale, float* state, long slot_stride,
                             const int* cu_tokens, const int* state_slots, const int* fresh, int n_seqs, int n_tokens,
                             int max_q_len, int heads, int key_dim, int value_dim, float* out, hipStream_t stream) {
  RA_CHECK(z && bias && cum && ldz >= heads * key_dim && tau > 0.f, "gla_chunks: pre-activation rows of %d for %d heads of %d, tau %g",
           ldz, heads, key_dim, tau);
  RA_CHECK(max_q_len > 0 && n_seqs <= 65535 && (max_q_len + CS_C - 1) / CS_C <= 65535, "gla_chunks: %d requests, portions up to %d",
           n_seqs, max_q_len);
  ChunkArgs a = {};
  a.n_seqs = n_seqs; a.H = heads; a.dk = key_dim; a.dv = value_dim;
  a.cu_tokens = cu_tokens; a.state_slots = state_slots; a.fresh = fresh; a.out = out;
  a.q_scale = q_scale; a.k_scale = 1.f; a.cum = cum;
  const int rc = chunk_common(a, "gla_chunks", 4, proj, act_dtype, ld, q_off, k_off, v_off, state, slot_stride, n_tokens);
  if (rc != 0) return rc;
  const int C = heads * key_dim;
  const dim3 grid((C + 255) / 256, (max_q_len + CS_C - 1) / CS_C, n_seqs);
  chunk_decay_kernel<<<grid, 256, 0, stream>>>(z, ldz, bias, 1.f / tau, cu_tokens, C, cum);
  RA_LAUNCH_CHECK("chunk_decay");
  return act_dtype == RA_F32 ? chunk_pick<float, CS_CHANNEL>(a, stream) : chunk_pick<bf16_t, CS_CHANNEL>(a, stream);
}
