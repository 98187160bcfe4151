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
