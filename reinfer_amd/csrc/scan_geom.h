// How the state of a recurrent mixer's head lies in a request's slot: shared by the kernel that walks a portion token
// by token and the one that takes it in chunks, so that either can go on from what the other left.
//
// R lanes share a column of the state, each holding a run of NPL of its elements; a wave holds CPW columns. Element e of
// column c of a head stands at
//   (head * waves + c / CPW) * wave_floats + (e % NPL) * 64 + (c % CPW) * R + e / NPL
// floats into the slot. R * NPL >= the key size; elements past it are zeros.
#pragma once
#include "common.h"

struct ScanGeom {
  int R, NPL, CPW, waves;      // lanes a column, elements a lane, columns a wave, waves a head
  int wave_floats;             // floats of state a wave
};

// kind 0: matrix memory (S, the normaliser n once a wave, the running maximum m); every other kind keeps S alone:
// 1 delta rule, 2 wkv, 3 a memory that fades by a constant a head, 4 gated linear attention
static inline bool scan_geom(int kind, int dk, int dv, ScanGeom* g) {
  if (dk <= 0 || dv <= 0 || dk > 512) return false;
  // at most 8 elements a lane: the per-token chain of multiply-adds stays short, and a head has enough waves to
  // spread over the chip when one request's prompt is all there is
  g->R = dk <= 32 ? 8 : dk <= 128 ? 16 : dk <= 256 ? 32 : 64;
  const int per = (dk + g->R - 1) / g->R;
  g->NPL = per <= 2 ? 2 : per <= 4 ? 4 : 8;
  g->CPW = RA_WAVE / g->R;
  g->waves = (dv + g->CPW - 1) / g->CPW;
  g->wave_floats = g->NPL * RA_WAVE + (kind == 0 ? g->NPL * g->R + 4 : 0);
  return true;
}

// log sigmoid without overflow
__device__ __forceinline__ float ra_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float ra_logsigmoid(float x) { return -ra_softplus(-x); }

// Sine and cosine of an angle (|x| up to 2^23), in few instructions and without branches: x less k times pi / 2, k the nearest
// whole number, pi / 2 in three parts (each step one fused multiply-add, whose product is exact), then the Taylor
// polynomials up to the 9th and 8th power on |r| <= pi / 4 (what they leave out is below 3e-8), swapped and signed by k's
// last two bits. Within 1.5e-7 of the exact values.
__device__ __forceinline__ void ra_sincos(float x, float* sn, float* cs) {
  const float k = rintf(x * 0.63661977236758134f);
  float r = fmaf(-k, 1.57079637050628662f, x);
  r = fmaf(-k, -4.37113882867379e-8f, r);
  r = fmaf(-k, -1.71512449e-15f, r);
  const float r2 = r * r;
  float s = fmaf(r2, 1.f / 362880.f, -1.f / 5040.f);
  s = fmaf(r2, s, 1.f / 120.f);
  s = fmaf(r2, s, -1.f / 6.f);
  s = fmaf(r * r2, s, r);
  float c = fmaf(r2, 1.f / 40320.f, -1.f / 720.f);
  c = fmaf(r2, c, 1.f / 24.f);
  c = fmaf(r2, c, -0.5f);
  c = fmaf(r2, c, 1.f);
  const int q = (int)k;
  const float a = (q & 1) ? c : s, b = (q & 1) ? s : c;
  *sn = (q & 2) ? -a : a;
  *cs = ((q + 1) & 2) ? -b : b;
}
