// Linear attention with a decay, a prompt's portion in chunks of 16 tokens on the float matrix cores.
//
//   S_t = A_t S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t          per head, S [dk, dv] float, from and into the request's slot
//
// with A_t one factor a head (a memory that fades by a constant, retention) or one a key channel and token (gated linear
// attention). Token by token this is a chain of as many steps as there are tokens; a chunk of C = 16 tokens is a handful
// of 16 x 16 products instead. With B_i the product of the factors from the chunk's first token to its i-th, S the state
// before the chunk:
//
//   o_i = (B_i q_i)^T S + sum_(j <= i) a_ij v_j,   a_ij = q_i . (B_i / B_j) k_j
//   S'  = B_C S + sum_j ((B_C / B_j) k_j) v_j^T
//
// Two kernels. chunk_prepare_kernel, one workgroup a (chunk, head), all chunks side by side: what lies between the
// projection and the recurrence (silu, or rotation and factors; the decays from their pre-activations), the scores a, and
// the factors; it leaves B_i q_i, (B_C / B_j) k_j, B_C, v and a as floats in the order in which the products want them.
// chunk_carry_kernel walks a request's chunks with nothing left to do but those products: a workgroup is one (request,
// head, 16 columns of v), its waves (four, or eight for keys above 64) split dk, the state stays in their accumulators
// from the portion's first chunk to its last, operands come straight from memory, CS_AHEAD chunks ahead.
//
// Everything is float: the products are v_mfma_f32_16x16x4_f32. The accumulator of a 16 x 16 product (row 4 g + i, column
// r in lane 16 g + r, register i) is at the same time the operand of a product over those rows, if step i of four takes
// rows {i, 4 + i, 8 + i, 12 + i}: so S is used where it lies. No factor is above 1 (for decays up to 1): B_i and
// B_C / B_j are formed as they stand; the scores are the product of B_i q_i with k_j / B_j where no channel falls below
// 2^-60 inside the chunk, else they are summed pair by pair with B_i / B_j, which never overflows.
//
// The state's layout in the slot is the token-by-token kernel's (scan_geom.h): steps may change from one to the other.
#include "common.h"
#include "reinfer_hip.h"
#include "scan_geom.h"

namespace {

#define CS_C 16                 // tokens of a chunk
#define CS_VP 20                // floats between rows of the waves' parts in LDS
#define CS_AHEAD 4              // chunks whose operands are on their way (a multiple of 4)
#define CS_LIMIT 60.f           // -log2 of the smallest factor that the product form of the scores takes

enum { CS_SILU = 0, CS_TURN = 1, CS_CHANNEL = 2 };       // silu on q, k, v; rotation and factors; a decay a key channel

struct ChunkArgs {
  const void* q; const void* k; const void* v;      // column 0 of each in row 0; rows ld elements apart
  int ld;
  float q_scale, k_scale;
  const int* positions; const float* inv_freq; int rot_dims;      // CS_TURN: the turn of q's and k's first elements
  const float* head_decay;                           // one factor a head
  const float* z; int ldz; const float* bias; float inv_tau;      // CS_CHANNEL: the decays' pre-activations
  float* state; long slot_stride;
  const int* cu_tokens; const int* state_slots; const int* fresh;
  int n_seqs, n_tokens, H, dk, dv, dkp, waves_per_head, wave_floats, R, NPL, CPW;
  int vec;                                           // rows of q and k in whole 16-byte pieces of 8 elements
  float* ops;                                        // the prepared operands
  float* out;                                        // [T][H dv]
};

// A request's chunks stand at places chunk_base(request) .. in the operands' buffer: portions of any length never overlap,
// and there are at most n_tokens / 16 + n_seqs places.
__host__ __device__ __forceinline__ long chunk_places(int n_tokens, int n_seqs) { return n_tokens / CS_C + n_seqs; }
__device__ __forceinline__ int chunk_base(const int* cu, int seq) { return cu[seq] / CS_C + seq; }
// Floats of one (chunk, head): q and k [dkp / 16 tiles][64 lanes][4], v [dv / 16 column groups][64][4], the scores
// [4 steps][64 lanes], B_C [dkp].
struct ChunkLayout { int k, v, a, b, floats; };
__host__ __device__ __forceinline__ ChunkLayout chunk_layout(int dkp, int dv) {
  ChunkLayout L;
  L.k = dkp * CS_C;
  L.v = 2 * dkp * CS_C;
  L.a = L.v + (dv + 15) / 16 * 256;
  L.b = L.a + 256;
  L.floats = L.b + dkp;
  return L;
}

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

template <typename TA, int MODE>
__global__ void __launch_bounds__(256) chunk_prepare_kernel(ChunkArgs p) {
  constexpr bool CHANNEL = MODE == CS_CHANNEL;
  extern __shared__ __attribute__((aligned(16))) float lds[];      // q, k and, a channel each, log2 B: [16][dkp + 4]
  const int dkp = p.dkp, pitch = dkp + 4, dk = p.dk;
  float* Q = lds;
  float* K = Q + CS_C * pitch;
  float* B = K + CS_C * pitch;
  float* red = CHANNEL ? B + CS_C * pitch : B;       // the waves' parts of the scores [4][16][CS_VP]
  const int tid = threadIdx.x, lane = tid & (RA_WAVE - 1), wave = tid / RA_WAVE;
  const int r = lane & 15, g = lane >> 4;
  const int place = blockIdx.x / p.H, head = blockIdx.x % p.H;
  int lo = 0, hi = p.n_seqs - 1;                     // the last request whose places start at or before this one
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (chunk_base(p.cu_tokens, mid) <= place) lo = mid;
    else hi = mid - 1;
  }
  const int t0 = p.cu_tokens[lo] + (place - chunk_base(p.cu_tokens, lo)) * CS_C, last = p.cu_tokens[lo + 1];
  if (t0 >= last || p.state_slots[lo] < 0) return;   // a place nobody has, or a padding row
  const int n = min(CS_C, last - t0);
  const ChunkLayout L = chunk_layout(dkp, p.dv);
  float* W = p.ops + ((size_t)place * p.H + head) * L.floats;
  const TA* qg = (const TA*)p.q + (size_t)t0 * p.ld + (size_t)head * dk;
  const TA* kg = (const TA*)p.k + (size_t)t0 * p.ld + (size_t)head * dk;
  const TA* vg = (const TA*)p.v + (size_t)t0 * p.ld + (size_t)head * p.dv;
  const int half = p.rot_dims >> 1;

  // ---- q and k of the chunk as floats
  const int segs = dkp / 8;
  for (int idx = tid; idx < CS_C * segs; idx += 256) {
    const int t = idx / segs, e = (idx % segs) * 8;
    float q8[8], k8[8], b8[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) q8[i] = k8[i] = b8[i] = 0.f;
    if (t < n && e < dk) {
      const size_t at = (size_t)t * p.ld + e;
      if (p.vec) {
        Vec8<TA>::load(qg + at, q8);
        Vec8<TA>::load(kg + at, k8);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i)
          if (e + i < dk) {
            q8[i] = to_f32(qg[at + i]);
            k8[i] = to_f32(kg[at + i]);
          }
      }
      if (MODE == CS_SILU) {
#pragma unroll
        for (int i = 0; i < 8; ++i) { q8[i] = silu_fast(q8[i]); k8[i] = silu_fast(k8[i]); }
      }
      if (CHANNEL) {
        const float* zp = p.z + (size_t)(t0 + t) * p.ldz + (size_t)head * dk + e;
        const float* bp = p.bias + (size_t)head * dk + e;
#pragma unroll
        for (int i = 0; i < 8; ++i)
          if (e + i < dk) b8[i] = ra_logsigmoid(zp[i] + bp[i]) * p.inv_tau * 1.4426950408889634f;
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) { q8[i] *= p.q_scale; k8[i] *= p.k_scale; }
    Vec8<float>::store(Q + t * pitch + e, q8);
    Vec8<float>::store(K + t * pitch + e, k8);
    if (CHANNEL) Vec8<float>::store(B + t * pitch + e, b8);
  }
  __syncthreads();
  if (MODE == CS_TURN && half > 0) {                 // a thread a pair, in place
    for (int idx = tid; idx < n * half; idx += 256) {
      const int t = idx / half, j = idx % half;
      float sn, cs;
      ra_sincos((float)p.positions[t0 + t] * p.inv_freq[j], &sn, &cs);
      float* q = Q + t * pitch + j;
      float* k = K + t * pitch + j;
      const float qa = q[0], qb = q[half], ka = k[0], kb = k[half];
      q[0] = qa * cs - qb * sn;
      q[half] = qb * cs + qa * sn;
      k[0] = ka * cs - kb * sn;
      k[half] = kb * cs + ka * sn;
    }
    __syncthreads();
  }
  if (CHANNEL) {                                     // log2 B: sums from the chunk's first token on
    for (int c = tid; c < dkp; c += 256) {
      float sum = 0.f;
#pragma unroll
      for (int t = 0; t < CS_C; ++t) {
        sum += B[t * pitch + c];                     // rows past n add nothing
        B[t * pitch + c] = sum;
      }
    }
    __syncthreads();
  }
  const float* BC = B + (CS_C - 1) * pitch;          // log2 B_C: rows past n repeat it

  // ---- the scores, transposed: a[i] is that of query r on key 4 g + i, the wave's part of dk
  const float d = CHANNEL ? 1.f : p.head_decay[head];
  const int tiles = dkp / 16, per = tiles / 4;       // dkp is a multiple of 64
  f32x4_t a = {0.f, 0.f, 0.f, 0.f};
  bool direct = false;
  if (CHANNEL) {
    float low = 0.f;
    for (int c = wave * per * 16 + lane; c < (wave + 1) * per * 16; c += RA_WAVE) low = fminf(low, BC[c]);
    direct = __any(!(low >= -CS_LIMIT));
  }
  if (!direct) {
    for (int nt = wave * per; nt < (wave + 1) * per; ++nt) {
      const int at = r * pitch + nt * 16 + 4 * g;
      f32x4_t q = *(const f32x4_t*)(Q + at), k = *(const f32x4_t*)(K + at);
      if (CHANNEL) {
        const f32x4_t b = *(const f32x4_t*)(B + at);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          q[i] *= __builtin_amdgcn_exp2f(b[i]);
          k[i] *= __builtin_amdgcn_exp2f(-b[i]);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) a = __builtin_amdgcn_mfma_f32_16x16x4f32(k[i], q[i], a, 0, 0, 0);
    }
  } else {
    for (int c = wave * per * 16; c < (wave + 1) * per * 16; ++c) {
      const float bq = B[r * pitch + c], qv = Q[r * pitch + c];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = 4 * g + i;
        a[i] += qv * K[j * pitch + c] * __builtin_amdgcn_exp2f(fminf(bq - B[j * pitch + c], 0.f));
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) red[(wave * CS_C + 4 * g + i) * CS_VP + r] = a[i];
  __syncthreads();
  {
    // thread: step `wave` of four, lane (r, g): query r on key 4 g + wave
    const int j = 4 * g + wave;
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) s += red[(w * CS_C + j) * CS_VP + r];
    W[L.a + tid] = r >= j ? s * (CHANNEL ? 1.f : power(d, r - j)) : 0.f;
  }

  // ---- operands in the products' order: a wave's lane (r, g) holds row r, columns 4 g + i of a tile of q, rows 4 g + i,
  // column r of one of k or v
  const float fq = CHANNEL ? 1.f : power(d, r + 1);
  float fk[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) fk[i] = CHANNEL ? 1.f : power(d, max(n - 1 - (4 * g + i), 0));      // rows past n are zeros
  for (int nt = wave; nt < tiles; nt += 4) {
    f32x4_t q = *(const f32x4_t*)(Q + r * pitch + nt * 16 + 4 * g), k;
    if (CHANNEL) {
      const f32x4_t b = *(const f32x4_t*)(B + r * pitch + nt * 16 + 4 * g);
#pragma unroll
      for (int i = 0; i < 4; ++i) q[i] *= __builtin_amdgcn_exp2f(b[i]);
    }
    const float bc = CHANNEL ? BC[nt * 16 + r] : 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int at = (4 * g + i) * pitch + nt * 16 + r;
      k[i] = K[at] * fk[i];
      if (CHANNEL) k[i] *= __builtin_amdgcn_exp2f(fminf(bc - B[at], 0.f));
      q[i] *= fq;
    }
    *(f32x4_t*)(W + (nt * RA_WAVE + lane) * 4) = q;
    *(f32x4_t*)(W + L.k + (nt * RA_WAVE + lane) * 4) = k;
    if (lane < 16) W[L.b + nt * 16 + r] = CHANNEL ? __builtin_amdgcn_exp2f(bc) : power(d, n);
  }
  for (int cg = wave; cg < (p.dv + 15) / 16; cg += 4) {
    const int col = cg * 16 + r;
    f32x4_t v;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * g + i;
      float x = (t < n && col < p.dv) ? to_f32(vg[(size_t)t * p.ld + col]) : 0.f;
      if (MODE == CS_SILU) x = silu_fast(x);
      v[i] = x;
    }
    *(f32x4_t*)(W + L.v + (cg * RA_WAVE + lane) * 4) = v;
  }
}

// NT: 16-row tiles of S a wave holds (dkp = 16 NT WAVES)
template <int NT, int WAVES>
__global__ void __launch_bounds__(WAVES * RA_WAVE) chunk_carry_kernel(ChunkArgs p) {
  constexpr int DKP = 16 * NT * WAVES, THREADS = WAVES * RA_WAVE;
  constexpr int PART = CS_C * CS_VP;                 // a wave's part of a chunk's o
  __shared__ float red[2][2][WAVES * PART];          // two chunks a barrier, two buffers
  const int tid = threadIdx.x, lane = tid & (RA_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(tid / RA_WAVE);
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
  float* out = p.out + (size_t)head * p.dv + cg * 16;
  const int cols = min(16, p.dv - cg * 16);
  if (slot < 0) {                                    // a padding row: no state, a defined result
    for (int idx = tid; idx < (last - first) * 16; idx += THREADS)
      if (idx % 16 < cols) out[(size_t)(first + idx / 16) * ow + idx % 16] = 0.f;
    return;
  }
  if (first >= last) return;
  const int n_chunks = (last - first + CS_C - 1) / CS_C;
  const ChunkLayout L = chunk_layout(DKP, p.dv);
  const size_t stride = (size_t)p.H * L.floats;      // from one chunk to the next
  const float* W = p.ops + (size_t)chunk_base(p.cu_tokens, seq) * stride + (size_t)head * L.floats;
  // Operands and results go through buffer descriptors, and no memory access stands under a condition: a store past the
  // descriptor's end is dropped, and with the same number of accesses on every path the waits for operands count exactly
  // those asked for (under a condition the compiler waited for all of them: one trip to memory every two chunks).
  const int q_at = (wave * NT * 256 + lane * 4) * 4, k_at = q_at + L.k * 4, b_at = (L.b + wave * NT * 16 + 4 * g) * 4;
  const int v_at = (L.v + cg * 256 + lane * 4) * 4, a_at = (L.a + (wave & 3) * RA_WAVE + lane) * 4;

  // ---- the state: tile nt of the wave is rows base + 16 nt + 4 g + i, column r of the group
  const int base = wave * 16 * NT, col = cg * 16 + r;
  const bool col_ok = r < cols;
  const int c_at = col_ok ? col : 0;
  float* st = p.state + (size_t)slot * p.slot_stride + ((size_t)head * p.waves_per_head + c_at / p.CPW) * p.wave_floats +
              (size_t)(c_at % p.CPW) * p.R;
  const bool from_zero = p.fresh[seq] != 0;
  f32x4_t S[NT], S_last[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = base + 16 * nt + 4 * g + i;
      S[nt][i] = (!from_zero && col_ok && e < p.dk) ? st[(size_t)(e % p.NPL) * RA_WAVE + e / p.NPL] : 0.f;
    }

  struct Operands { f32x4_t q[NT], k[NT], b[NT], v; float a; };
  auto load = [&](int c, Operands& x) {              // a chunk past the last reads the last one again
    const __amdgpu_buffer_rsrc_t rsrc = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<float*>(W + (size_t)min(c, n_chunks - 1) * stride), 0, L.floats * 4, 0x00020000);
    auto four = [&](int at) { return __builtin_bit_cast(f32x4_t, __builtin_amdgcn_raw_buffer_load_b128(rsrc, at, 0, 0)); };
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      x.q[nt] = four(q_at + nt * 1024);
      x.k[nt] = four(k_at + nt * 1024);
      x.b[nt] = four(b_at + nt * 64);
    }
    x.v = four(v_at);
    x.a = __builtin_bit_cast(float, __builtin_amdgcn_raw_buffer_load_b32(rsrc, a_at, 0, 0));
  };
  auto step = [&](int c, const Operands& x, float* part) {
    f32x4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[nt][i], S[nt][i], o, 0, 0, 0);
    if (wave < 4) {                                  // the first four waves add a step of scores times v each
      const float v = wave == 0 ? x.v[0] : wave == 1 ? x.v[1] : wave == 2 ? x.v[2] : x.v[3];
      o = __builtin_amdgcn_mfma_f32_16x16x4f32(x.a, v, o, 0, 0, 0);
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
#pragma unroll
      for (int i = 0; i < 4; ++i) S[nt][i] *= x.b[nt][i];
#pragma unroll
      for (int i = 0; i < 4; ++i) S[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[nt][i], x.v[i], S[nt], 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) S_last[nt][i] = c < n_chunks ? S[nt][i] : S_last[nt][i];      // a chunk past the last leaves no trace
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave * PART + (4 * g + i) * CS_VP + r] = o[i];
  };
  // where this thread's elements of two chunks' o go, in a window of rows that begins at the first of the two
  int o_at[512 / THREADS];
#pragma unroll
  for (int u = 0; u < 512 / THREADS; ++u) {
    const int idx = tid + u * THREADS, t = idx / 16, e = idx % 16;
    o_at[u] = e < cols ? (int)((t * ow + e) * 4) : -1;
  }
  // two chunks a barrier; every set of operands is asked for CS_AHEAD chunks before its use
  auto round = [&](int c, Operands& xa, Operands& xb, int buf) {
    step(c, xa, red[buf][0]);
    load(c + CS_AHEAD, xa);
    __builtin_amdgcn_sched_barrier(0);               // the loads stay where they are asked for
    step(c + 1, xb, red[buf][1]);
    load(c + 1 + CS_AHEAD, xb);
    __builtin_amdgcn_sched_barrier(0);
    __syncthreads();
    // a thread an element of o: the waves' parts in order. The next round writes the other buffer, and the one after it
    // this one again, behind a barrier that every thread reaches only after its reads here.
    const int row0 = min(first + c * CS_C, last), rows = min(2 * CS_C, last - row0);
    const __amdgpu_buffer_rsrc_t rsrc =
        __builtin_amdgcn_make_buffer_rsrc(out + (size_t)row0 * ow, 0, (int)(rows * ow * 4), 0x00020000);
#pragma unroll
    for (int u = 0; u < 512 / THREADS; ++u) {
      const int idx = tid + u * THREADS, t = idx / 16, e = idx % 16;
      const float* part = red[buf][t / CS_C] + (t % CS_C) * CS_VP + e;
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) s += part[w * PART];
      __builtin_amdgcn_raw_buffer_store_b32(__builtin_bit_cast(unsigned, s), rsrc, o_at[u], 0, 0);
    }
  };
  Operands x[CS_AHEAD];
#pragma unroll
  for (int k = 0; k < CS_AHEAD; ++k) {
    load(k, x[k]);
    __builtin_amdgcn_sched_barrier(0);
  }
  for (int c = 0; c < n_chunks; c += CS_AHEAD) {
#pragma unroll
    for (int k = 0; k < CS_AHEAD; k += 2)
      round(c + k, x[k], x[k + 1], (k >> 1) & 1);
  }
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = base + 16 * nt + 4 * g + i;
      if (col_ok && e < p.R * p.NPL) st[(size_t)(e % p.NPL) * RA_WAVE + e / p.NPL] = S_last[nt][i];
    }
}

int chunk_dkp(const ScanGeom& g) { return g.R * g.NPL <= 64 ? 64 : g.R * g.NPL <= 128 ? 128 : 256; }

template <typename TA, int MODE>
int chunk_run(const ChunkArgs& a, const char* what, hipStream_t stream) {
  const long places = chunk_places(a.n_tokens, a.n_seqs) * a.H;
  const long units = ((long)a.n_seqs * a.H + RA_XCDS - 1) / RA_XCDS * RA_XCDS * ((a.dv + 15) / 16);
  RA_CHECK(places <= 0x7fffffffL && units <= 0x7fffffffL, "%s: too many workgroups", what);
  const size_t lds = (size_t)(CS_C * (a.dkp + 4) * (MODE == CS_CHANNEL ? 3 : 2) + 4 * CS_C * CS_VP) * sizeof(float);
  RA_CHECK(lds <= 64 * 1024, "%s: %zu bytes of LDS", what, lds);
  RA_CHECK((long)a.H * a.dv * 2 * CS_C * 4 < (1L << 31), "%s: rows of %ld floats", what, (long)a.H * a.dv);
  chunk_prepare_kernel<TA, MODE><<<(unsigned)places, 256, lds, stream>>>(a);
  RA_LAUNCH_CHECK(what);
  if (a.dkp == 64) chunk_carry_kernel<1, 4><<<(unsigned)units, 4 * RA_WAVE, 0, stream>>>(a);
  else if (a.dkp == 128) chunk_carry_kernel<1, 8><<<(unsigned)units, 8 * RA_WAVE, 0, stream>>>(a);
  else chunk_carry_kernel<2, 8><<<(unsigned)units, 8 * RA_WAVE, 0, stream>>>(a);
  RA_LAUNCH_CHECK(what);
  return 0;
}

int chunk_common(ChunkArgs& a, const char* what, int kind, const void* proj, int act_dtype, int ld, int q_off, int k_off,
                 int v_off, float* state, long slot_stride, long scratch) {
  RA_CHECK(a.n_seqs > 0 && a.n_tokens > 0 && a.H > 0, "%s: %d requests, %d tokens, %d heads", what, a.n_seqs, a.n_tokens, a.H);
  RA_CHECK(act_dtype == RA_F32 || act_dtype == RA_BF16, "%s: unknown dtype tag %d", what, act_dtype);
  ScanGeom g;
  RA_CHECK(scan_geom(kind, a.dk, a.dv, &g) && a.dk <= 256, "%s: heads of %d x %d (keys up to 256)", what, a.dk, a.dv);
  RA_CHECK(slot_stride >= (long)a.H * g.waves * g.wave_floats, "%s: a state slot of %ld floats, need %ld", what, slot_stride,
           (long)a.H * g.waves * g.wave_floats);
  const long need = ra_chunk_scratch_floats(a.n_tokens, a.n_seqs, a.H, a.dk, a.dv);
  RA_CHECK(a.ops != nullptr && ((uintptr_t)a.ops % 16) == 0 && scratch >= need, "%s: %ld floats of scratch, need %ld, 16-byte aligned",
           what, scratch, need);
  const size_t es = act_dtype == RA_F32 ? 4 : 2;
  a.q = (const char*)proj + (size_t)q_off * es;
  a.k = (const char*)proj + (size_t)k_off * es;
  a.v = (const char*)proj + (size_t)v_off * es;
  a.ld = ld; a.state = state; a.slot_stride = slot_stride; a.dkp = chunk_dkp(g);
  a.waves_per_head = g.waves; a.wave_floats = g.wave_floats; a.R = g.R; a.NPL = g.NPL; a.CPW = g.CPW;
  a.vec = a.dk % 8 == 0 && ((long)ld * es) % 16 == 0 && ((uintptr_t)a.q % 16) == 0 && ((uintptr_t)a.k % 16) == 0;
  return 0;
}

}  // namespace

// Floats of scratch that a call of ra_decay_chunks or ra_gla_chunks needs; -1 for heads that they do not take.
extern "C" long ra_chunk_scratch_floats(int n_tokens, int n_seqs, int heads, int key_dim, int value_dim) {
  ScanGeom g;
  if (n_tokens <= 0 || n_seqs <= 0 || heads <= 0 || !scan_geom(3, key_dim, value_dim, &g) || key_dim > 256) return -1;
  return chunk_places(n_tokens, n_seqs) * heads * chunk_layout(chunk_dkp(g), value_dim).floats;
}

// The recurrence of ra_decay_scan (silu) and ra_retention_scan in chunks, for steps with portions; the same state.
extern "C" int ra_decay_chunks(const void* proj, int act_dtype, int ld, int q_off, int k_off, int v_off, int silu,
                               const float* decays, const int* positions, const float* inv_freq, int rot_dims,
                               float q_scale, float k_scale, float* state, long slot_stride, const int* cu_tokens,
                               const int* state_slots, const int* fresh, int n_seqs, int n_tokens, int heads, int key_dim,
                               int value_dim, float* scratch, long scratch_floats, float* out, hipStream_t stream) {
  RA_CHECK(decays != nullptr, "decay_chunks: one factor a head is needed");
  RA_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= key_dim && (rot_dims == 0 || (positions && inv_freq && !silu)),
           "decay_chunks: %d turned elements of %d", rot_dims, key_dim);
  ChunkArgs a = {};
  a.n_seqs = n_seqs; a.n_tokens = n_tokens; a.H = heads; a.dk = key_dim; a.dv = value_dim;
  a.cu_tokens = cu_tokens; a.state_slots = state_slots; a.fresh = fresh; a.ops = scratch; a.out = out;
  a.q_scale = q_scale; a.k_scale = k_scale; a.head_decay = decays;
  a.positions = positions; a.inv_freq = inv_freq; a.rot_dims = rot_dims;
  const int rc = chunk_common(a, "decay_chunks", 3, proj, act_dtype, ld, q_off, k_off, v_off, state, slot_stride, scratch_floats);
  if (rc != 0) return rc;
  if (silu) return act_dtype == RA_F32 ? chunk_run<float, CS_SILU>(a, "decay_chunks", stream) : chunk_run<bf16_t, CS_SILU>(a, "decay_chunks", stream);
  return act_dtype == RA_F32 ? chunk_run<float, CS_TURN>(a, "decay_chunks", stream) : chunk_run<bf16_t, CS_TURN>(a, "decay_chunks", stream);
}

// The recurrence of ra_gla_scan in chunks.
extern "C" int ra_gla_chunks(const void* proj, int act_dtype, int ld, int q_off, int k_off, int v_off, const float* z, int ldz,
                             const float* bias, float tau, float q_scale, float* state, long slot_stride,
                             const int* cu_tokens, const int* state_slots, const int* fresh, int n_seqs, int n_tokens,
                             int heads, int key_dim, int value_dim, float* scratch, long scratch_floats, float* out,
                             hipStream_t stream) {
  RA_CHECK(z && bias && ldz >= heads * key_dim && tau > 0.f, "gla_chunks: pre-activation rows of %d for %d heads of %d, tau %g",
           ldz, heads, key_dim, tau);
  ChunkArgs a = {};
  a.n_seqs = n_seqs; a.n_tokens = n_tokens; a.H = heads; a.dk = key_dim; a.dv = value_dim;
  a.cu_tokens = cu_tokens; a.state_slots = state_slots; a.fresh = fresh; a.ops = scratch; a.out = out;
  a.q_scale = q_scale; a.k_scale = 1.f; a.z = z; a.ldz = ldz; a.bias = bias; a.inv_tau = 1.f / tau;
  const int rc = chunk_common(a, "gla_chunks", 4, proj, act_dtype, ld, q_off, k_off, v_off, state, slot_stride, scratch_floats);
  if (rc != 0) return rc;
  return act_dtype == RA_F32 ? chunk_run<float, CS_CHANNEL>(a, "gla_chunks", stream) : chunk_run<bf16_t, CS_CHANNEL>(a, "gla_chunks", stream);
}
