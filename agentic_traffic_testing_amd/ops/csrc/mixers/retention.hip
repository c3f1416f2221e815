// Retention: linear attention with one fixed decay g per head over ragged batches of portions, state
// carried per sequence in fp32.
//
// Per head, with S [dk, dv] the state, per token:   S = g S + k v^T,   o = S^T q
// q and k are rotated here (rotate-half pairs (i, i + n_freq) over the first 2 n_freq channels,
// cos / sin from the step's table) and k times dk^-1/2, so everything after the projections is fp32.
//
// * chunk kernel (portions; dk <= 128): since g does not depend on the data, C = 64 tokens at a time
//   are matrix products, with S the state before the chunk and tokens counted from its start:
//     o_i = g^(i+1) S^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j
//     S   = g^n S + sum_j g^(n-1-j) k_j v_j^T            (n tokens in the chunk)
//   A workgroup of four waves owns 64 value columns of one (sequence, head) and walks its chunks;
//   all products run on the fp32 matrix instructions (32x32x2), so nothing is rounded to 16 bits
//   on the way.  Wave w computes one 32 x 32 block of the masked scores (as P^T, so a lane writes
//   four neighbours of a row of P), one of the output, and holds dk / 64 blocks of S in its
//   accumulators for the whole portion; S goes through LDS once per chunk as the next chunk's
//   operand.  Operands whose K dimension is contiguous in LDS are read 16 bytes at a time: inside
//   8 K values lane half h takes 4 h ... 4 h + 3, which both operands agree on.  The raw rows of
//   the next chunk are fetched into registers while the current chunk's products run.
// * step kernel (decode rows; any dk <= 256): a workgroup owns 64 value columns of one (sequence,
//   head); 16 row groups x 16 lanes of 4 adjacent columns hold S in registers (coalesced state
//   I/O), tokens one by one.
// A portion whose first position is 0 starts from the zero state whatever its slot holds.
#include "mix_common.h"
#include "mixers.h"

namespace mixk {

constexpr int kChunk = 64;
constexpr int kRetCols = 64;       // value columns per workgroup
constexpr int kTokStride = kChunk + 4;
typedef __attribute__((ext_vector_type(16))) float rf32x16;
typedef __attribute__((ext_vector_type(4))) float rf32x4;

struct RetArgs {
  float* out;             // [T, H, dv]
  float* state;           // [slots, H, dk, dv]
  const void* q;          // [T, H dk]
  const void* k;          // [T, H dk]
  const void* v;          // [T, H dv]
  const float* powers;    // [H, kChunk + 1]: g^0 ... g^kChunk
  const float* cos_sin;   // [T, 2 n_freq]
  const int* positions;
  const int* seq_qstart;
  const int* seq_slot;
  int64_t q_stride, k_stride, v_stride;
  int H, dk, dv, n_freq, seq0;   // seq0: sequence of blockIdx.x 0
  float kscale;
};

// channels of pair p of a head: (p, p + n_freq) while they rotate, neighbours after that
__device__ __forceinline__ int pair_a(int p, int n_freq) { return p < n_freq ? p : 2 * p; }
__device__ __forceinline__ int pair_b(int p, int n_freq) { return p < n_freq ? p + n_freq : 2 * p + 1; }

__device__ __forceinline__ rf32x16 mfma_f32(float a, float b, rf32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x2f32(a, b, c, 0, 0, 0);
}

// DK: key width padded to 32, 64 or 128.  VEC: 8 channels per load (dk % 16, dv % 8, n_freq % 8 == 0,
// aligned rows); a group of 8 pairs then is 8 + 8 adjacent channels.
template <typename T, int DK, bool VEC>
__global__ void __launch_bounds__(256, 1)
retention_chunk_kernel(RetArgs a) {
  constexpr int DS = DK + 4;                    // LDS row of q, k and S^T
  constexpr int NDB = DK / 32;                  // 32-row blocks of S
  constexpr int SB = (2 * NDB + 3) / 4;         // blocks of S per wave
  constexpr int PG = DK / 16;                   // groups of 8 pairs per token
  constexpr int NI = (kChunk * PG + 255) / 256; // (token, group) items per thread
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* Qs = lds;                              // [64][DS]
  float* Ks = Qs + kChunk * DS;                 // [64][DS]
  float* St = Ks + kChunk * DS;                 // [64 columns][DS]: S^T
  float* Vt = St + kRetCols * DS;               // [64 columns][kTokStride]: V^T
  float* Vd = Vt + kRetCols * kTokStride;       // the same, decayed to the end of the chunk
  float* Ps = Vd + kRetCols * kTokStride;       // [64][kTokStride]: masked, decayed scores
  float* pw = Ps + kChunk * kTokStride;         // [kChunk + 1]
  const int s = a.seq0 + blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = a.seq_slot[s];
  const int first = a.seq_qstart[s], n = a.seq_qstart[s + 1] - first;
  if (slot < 0 || n <= 0) return;
  const int dk = a.dk, dv = a.dv, H = a.H, n_freq = a.n_freq;
  const int lane = tid & 63, w = tid >> 6, r = lane & 31, hf = lane >> 5;
  const int c0 = blockIdx.z * kRetCols;
  const T* qp = static_cast<const T*>(a.q) + static_cast<int64_t>(h) * dk;
  const T* kp = static_cast<const T*>(a.k) + static_cast<int64_t>(h) * dk;
  const T* vp = static_cast<const T*>(a.v) + static_cast<int64_t>(h) * dv + c0;
  float* st = a.state + (static_cast<int64_t>(slot) * H + h) * dk * dv;
  if (tid <= kChunk) pw[tid] = a.powers[h * (kChunk + 1) + tid];
  // channels past dk stay zero in every staged array (V's columns past dv are staged as zeros)
  for (int i = tid; i < kChunk * DS; i += 256) Qs[i] = Ks[i] = St[i] = 0.f;
  // this wave's blocks of S: rows db 32 .. + 31, columns cb 32 .. + 31
  rf32x16 S[SB];
  const bool fresh = a.positions[first] == 0;
#pragma unroll
  for (int b = 0; b < SB; ++b) {
    const int blk = w + 4 * b, db = blk % NDB, col = c0 + (blk / NDB) * 32 + r;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = db * 32 + 8 * (i >> 2) + 4 * hf + (i & 3);
      S[b][i] = (!fresh && blk < 2 * NDB && d < dk && col < dv)
                    ? st[static_cast<int64_t>(d) * dv + col] : 0.f;
    }
  }
  __syncthreads();
  auto put_state = [&]() {
#pragma unroll
    for (int b = 0; b < SB; ++b) {
      const int blk = w + 4 * b, db = blk % NDB, cl = (blk / NDB) * 32 + r;
      if (blk < 2 * NDB)
#pragma unroll
        for (int i4 = 0; i4 < 4; ++i4)
          *reinterpret_cast<rf32x4*>(St + cl * DS + db * 32 + 8 * i4 + 4 * hf) =
              rf32x4{S[b][4 * i4], S[b][4 * i4 + 1], S[b][4 * i4 + 2], S[b][4 * i4 + 3]};
    }
  };
  put_state();
  // raw rows of a chunk, fetched one chunk ahead: q and k pairs of (token, group) items, cos / sin,
  // and V of (token, 8-column group) items (tokens across lanes: the transposing LDS writes are
  // then free of bank conflicts)
  T rqa[NI][8], rqb[NI][8], rka[NI][8], rkb[NI][8], rv[2][8];
  float rc[NI][8], rs[NI][8];
  auto load8 = [&](const T* p, T (&o)[8]) {
    if constexpr (sizeof(T) == 2) {
      *reinterpret_cast<bf16x8_t*>(o) = *reinterpret_cast<const bf16x8_t*>(p);
    } else {
      *reinterpret_cast<rf32x4*>(o) = *reinterpret_cast<const rf32x4*>(p);
      *reinterpret_cast<rf32x4*>(o + 4) = *reinterpret_cast<const rf32x4*>(p + 4);
    }
  };
  auto fetch = [&](int t0) {
#pragma unroll
    for (int m = 0; m < NI; ++m) {
      const int it = tid + m * 256, tt = it / PG, p0 = (it % PG) * 8;
      const bool live = it < kChunk * PG && t0 + tt < n;
      const int64_t row = first + t0 + (live ? tt : 0);
      const float* tab = a.cos_sin + row * 2 * n_freq;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        rqa[m][e] = rqb[m][e] = rka[m][e] = rkb[m][e] = static_cast<T>(0.f);
        rc[m][e] = 1.f;
        rs[m][e] = 0.f;
      }
      if (!live) continue;
      if (VEC) {
        const int ca = pair_a(p0, n_freq), cb = p0 < n_freq ? p0 + n_freq : ca + 8;
        if (2 * p0 < dk) {   // dk % 16 == 0: the whole group is in
          load8(qp + row * a.q_stride + ca, rqa[m]);
          load8(qp + row * a.q_stride + cb, rqb[m]);
          load8(kp + row * a.k_stride + ca, rka[m]);
          load8(kp + row * a.k_stride + cb, rkb[m]);
          if (p0 < n_freq) {
            ld8(tab + p0, rc[m]);
            ld8(tab + n_freq + p0, rs[m]);
          }
        }
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int p = p0 + e, ca = pair_a(p, n_freq), cb = pair_b(p, n_freq);
          if (ca < dk) {
            rqa[m][e] = qp[row * a.q_stride + ca];
            rka[m][e] = kp[row * a.k_stride + ca];
          }
          if (cb < dk) {
            rqb[m][e] = qp[row * a.q_stride + cb];
            rkb[m][e] = kp[row * a.k_stride + cb];
          }
          if (p < n_freq) {
            rc[m][e] = tab[p];
            rs[m][e] = tab[n_freq + p];
          }
        }
      }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int it = tid + m * 256, tt = it & 63, cg = (it >> 6) * 8;
      const bool live = t0 + tt < n;
      const int64_t row = first + t0 + (live ? tt : 0);
#pragma unroll
      for (int e = 0; e < 8; ++e) rv[m][e] = static_cast<T>(0.f);
      if (!live) continue;
      if (VEC) {
        if (c0 + cg < dv) load8(vp + row * a.v_stride + cg, rv[m]);
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (c0 + cg + e < dv) rv[m][e] = vp[row * a.v_stride + cg + e];
      }
    }
  };
  fetch(0);
  const int tb = w & 1, cb = w >> 1;   // output block: tokens tb 32 .., columns cb 32 ..
  for (int t0 = 0; t0 < n; t0 += kChunk) {
    const int nt = min(kChunk, n - t0);
    if (t0 > 0) __syncthreads();   // the previous chunk's reads of Ks / Vt / Ps are done
#pragma unroll
    for (int m = 0; m < NI; ++m) {
      const int it = tid + m * 256, tt = it / PG, p0 = (it % PG) * 8;
      if (it < kChunk * PG) {
        float qa[8], qb[8], ka[8], kb[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float ua = static_cast<float>(rqa[m][e]), ub = static_cast<float>(rqb[m][e]);
          const float xa = static_cast<float>(rka[m][e]), xb = static_cast<float>(rkb[m][e]);
          qa[e] = ua * rc[m][e] - ub * rs[m][e];
          qb[e] = ub * rc[m][e] + ua * rs[m][e];
          ka[e] = (xa * rc[m][e] - xb * rs[m][e]) * a.kscale;
          kb[e] = (xb * rc[m][e] + xa * rs[m][e]) * a.kscale;
        }
        if (VEC) {
          const int ca = pair_a(p0, n_freq), cbb = p0 < n_freq ? p0 + n_freq : ca + 8;
          if (2 * p0 < dk) {
            st8(Qs + tt * DS + ca, qa);
            st8(Qs + tt * DS + cbb, qb);
            st8(Ks + tt * DS + ca, ka);
            st8(Ks + tt * DS + cbb, kb);
          }
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int p = p0 + e, ca = pair_a(p, n_freq), cbb = pair_b(p, n_freq);
            if (ca < dk) {
              Qs[tt * DS + ca] = qa[e];
              Ks[tt * DS + ca] = ka[e];
            }
            if (cbb < dk) {
              Qs[tt * DS + cbb] = qb[e];
              Ks[tt * DS + cbb] = kb[e];
            }
          }
        }
      }
    }
    const float decay_to_end = pw[max(nt - 1 - (tid & 63), 0)];   // of this thread's V token
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int it = tid + m * 256, tt = it & 63, cg = (it >> 6) * 8;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float v = static_cast<float>(rv[m][e]);
        Vt[(cg + e) * kTokStride + tt] = v;
        Vd[(cg + e) * kTokStride + tt] = v * decay_to_end;
      }
    }
    __syncthreads();
    if (t0 + kChunk < n) fetch(t0 + kChunk);   // in flight during the products below
    // P^T block: rows j (keys) of half cb, columns i (queries) of half tb; j > i everywhere when
    // cb > tb
    if (cb <= tb) {
      rf32x16 P;
#pragma unroll
      for (int i = 0; i < 16; ++i) P[i] = 0.f;
      const float* kr = Ks + (cb * 32 + r) * DS + 4 * hf;
      const float* qr = Qs + (tb * 32 + r) * DS + 4 * hf;
#pragma unroll
      for (int d = 0; d < DK; d += 8) {
        const rf32x4 ka = *reinterpret_cast<const rf32x4*>(kr + d);
        const rf32x4 qa = *reinterpret_cast<const rf32x4*>(qr + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) P = mfma_f32(ka[e], qa[e], P);
      }
      const int i = tb * 32 + r;
#pragma unroll
      for (int i4 = 0; i4 < 4; ++i4) {
        const int j0 = cb * 32 + 8 * i4 + 4 * hf;
        rf32x4 x;
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = j0 + e <= i ? P[4 * i4 + e] * pw[max(i - j0 - e, 0)] : 0.f;
        *reinterpret_cast<rf32x4*>(Ps + i * kTokStride + j0) = x;
      }
    }
    // output block, part of the state: rows i (tokens), columns c
    rf32x16 O;
#pragma unroll
    for (int i = 0; i < 16; ++i) O[i] = 0.f;
    {
      const float* qr = Qs + (tb * 32 + r) * DS + 4 * hf;
      const float* sr = St + (cb * 32 + r) * DS + 4 * hf;
#pragma unroll
      for (int d = 0; d < DK; d += 8) {
        const rf32x4 qa = *reinterpret_cast<const rf32x4*>(qr + d);
        const rf32x4 sa = *reinterpret_cast<const rf32x4*>(sr + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) O = mfma_f32(qa[e], sa[e], O);
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) O[i] *= pw[tb * 32 + 8 * (i >> 2) + 4 * hf + (i & 3) + 1];
    }
    __syncthreads();   // P is written, S^T is read
    {
      const float* pr = Ps + (tb * 32 + r) * kTokStride + 4 * hf;
      const float* vr = Vt + (cb * 32 + r) * kTokStride + 4 * hf;
      const int jend = 32 * (tb + 1);
#pragma unroll
      for (int j = 0; j < kChunk; j += 8) {
        if (j < jend) {
          const rf32x4 pa = *reinterpret_cast<const rf32x4*>(pr + j);
          const rf32x4 va = *reinterpret_cast<const rf32x4*>(vr + j);
#pragma unroll
          for (int e = 0; e < 4; ++e) O = mfma_f32(pa[e], va[e], O);
        }
      }
      const int col = c0 + cb * 32 + r;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int tok = tb * 32 + 8 * (i >> 2) + 4 * hf + (i & 3);
        if (tok < nt && col < dv)
          a.out[(static_cast<int64_t>(first + t0 + tok) * H + h) * dv + col] = O[i];
      }
    }
    // state: S = g^nt S + K^T (decayed V); K columns are read one value per lane
    const float gn = pw[nt];
#pragma unroll
    for (int b = 0; b < SB; ++b)
#pragma unroll
      for (int i = 0; i < 16; ++i) S[b][i] *= gn;
#pragma unroll
    for (int b = 0; b < SB; ++b) {
      const int blk = w + 4 * b, db = blk % NDB, sc = blk / NDB;
      if (blk < 2 * NDB) {   // wave-uniform
        const float* kr = Ks + (4 * hf) * DS + db * 32 + r;
        const float* vr = Vd + (sc * 32 + r) * kTokStride + 4 * hf;
#pragma unroll
        for (int j = 0; j < kChunk; j += 8) {
          const rf32x4 va = *reinterpret_cast<const rf32x4*>(vr + j);
#pragma unroll
          for (int e = 0; e < 4; ++e) S[b] = mfma_f32(kr[(j + e) * DS], va[e], S[b]);
        }
      }
    }
    put_state();   // read again only after the next chunk's staging barrier
  }
#pragma unroll
  for (int b = 0; b < SB; ++b) {
    const int blk = w + 4 * b, db = blk % NDB, col = c0 + (blk / NDB) * 32 + r;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int d = db * 32 + 8 * (i >> 2) + 4 * hf + (i & 3);
      if (blk < 2 * NDB && d < dk && col < dv) st[static_cast<int64_t>(d) * dv + col] = S[b][i];
    }
  }
}

// R: rows of S per thread (dk <= 16 R); V4: 16-byte state I/O (dv % 4 == 0, aligned state).
template <typename T, int R, bool V4>
__global__ void __launch_bounds__(256)
retention_step_kernel(RetArgs a) {
  __shared__ float sq[256], sk[256];
  __shared__ float part[4][kRetCols];
  const int s = a.seq0 + blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = a.seq_slot[s];
  const int first = a.seq_qstart[s], n = a.seq_qstart[s + 1] - first;
  if (slot < 0 || n <= 0) return;
  const int dk = a.dk, dv = a.dv, H = a.H, n_freq = a.n_freq;
  const int cl = (tid & 15) * 4, rg = tid >> 4, col = blockIdx.z * kRetCols + cl;
  float* st = a.state + (static_cast<int64_t>(slot) * H + h) * dk * dv;
  const float g = a.powers[h * (kChunk + 1) + 1];
  const bool fresh = a.positions[first] == 0;
  sq[tid] = sk[tid] = 0.f;   // channels past dk stay zero: the token loop needs no bounds check
  rf32x4 S[R];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    // clamped addresses and a select: every load is in bounds and issued without a branch
    const int d = rg + 16 * j;
    const float* p = st + static_cast<int64_t>(min(d, dk - 1)) * dv;
    if (V4) S[j] = *reinterpret_cast<const rf32x4*>(p + min(col, dv - 4));
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      if (!V4) S[j][e] = p[min(col + e, dv - 1)];
      S[j][e] = !fresh && d < dk && col + e < dv ? S[j][e] : 0.f;
    }
  }
#pragma unroll 1
  for (int t = 0; t < n; ++t) {
    const int64_t row = first + t;
    const T* qr = static_cast<const T*>(a.q) + row * a.q_stride + static_cast<int64_t>(h) * dk;
    const T* kr = static_cast<const T*>(a.k) + row * a.k_stride + static_cast<int64_t>(h) * dk;
    const T* vr = static_cast<const T*>(a.v) + row * a.v_stride + static_cast<int64_t>(h) * dv;
    const float* tab = a.cos_sin + row * 2 * n_freq;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = col + e < dv ? ldf(vr + col + e) : 0.f;
    __syncthreads();   // the previous token's reads of sq / sk / part (or the fill above) are done
    if (tid < 128 && 2 * tid < dk + 1) {
      const int ca = pair_a(tid, n_freq), cb = pair_b(tid, n_freq);
      const float cs = tid < n_freq ? tab[tid] : 1.f, sn = tid < n_freq ? tab[n_freq + tid] : 0.f;
      if (ca < dk) {
        const float qa = ldf(qr + ca), ka = ldf(kr + ca);
        const float qb = cb < dk ? ldf(qr + cb) : 0.f, kb = cb < dk ? ldf(kr + cb) : 0.f;
        sq[ca] = qa * cs - qb * sn;
        sk[ca] = (ka * cs - kb * sn) * a.kscale;
        if (cb < dk) {
          sq[cb] = qb * cs + qa * sn;
          sk[cb] = (kb * cs + ka * sn) * a.kscale;
        }
      }
    }
    __syncthreads();
    float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < R; ++j) {
      const float kd = sk[rg + 16 * j], qd = sq[rg + 16 * j];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j][e] = g * S[j][e] + kd * v[e];
        o[e] += qd * S[j][e];
      }
    }
    // over the four row groups of the wave, then over the waves
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[e] += __shfl_xor(o[e], 16, kWave);
      o[e] += __shfl_xor(o[e], 32, kWave);
    }
    if ((tid & 63) < 16)
#pragma unroll
      for (int e = 0; e < 4; ++e) part[tid >> 6][cl + e] = o[e];
    __syncthreads();
    if (tid < kRetCols && blockIdx.z * kRetCols + tid < dv)
      a.out[(row * H + h) * dv + blockIdx.z * kRetCols + tid] =
          part[0][tid] + part[1][tid] + part[2][tid] + part[3][tid];
  }
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int d = rg + 16 * j;
    if (d < dk) {
      float* p = st + static_cast<int64_t>(d) * dv + col;
      if (V4) {
        if (col < dv) *reinterpret_cast<rf32x4*>(p) = S[j];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (col + e < dv) p[e] = S[j][e];
      }
    }
  }
}

template <typename T, int DK, bool VEC>
int launch_chunk(const RetArgs& a, int seqs, hipStream_t st) {
  constexpr size_t smem = sizeof(float) * (3 * kChunk * (DK + 4) + 3 * kChunk * kTokStride + kChunk + 4);
  static bool opted = false;
  if (smem > 48 * 1024 && !opted) {
    hipError_t e = hipFuncSetAttribute(
        reinterpret_cast<const void*>(&retention_chunk_kernel<T, DK, VEC>),
        hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(smem));
    if (e != hipSuccess) return static_cast<int>(e);
    opted = true;
  }
  hipLaunchKernelGGL((retention_chunk_kernel<T, DK, VEC>),
                     dim3(seqs, a.H, (a.dv + kRetCols - 1) / kRetCols), dim3(256), smem, st, a);
  return static_cast<int>(hipGetLastError());
}

template <typename T, bool V4>
int launch_step(const RetArgs& a, int seqs, hipStream_t st) {
  const dim3 grid(seqs, a.H, (a.dv + kRetCols - 1) / kRetCols);
#define MIXK_STEP(R)                                                                               \
  if (a.dk <= 16 * R) {                                                                            \
    hipLaunchKernelGGL((retention_step_kernel<T, R, V4>), grid, dim3(256), 0, st, a);              \
    return static_cast<int>(hipGetLastError());                                                    \
  }
  MIXK_STEP(4)
  MIXK_STEP(8)
  MIXK_STEP(16)
#undef MIXK_STEP
  return -1;
}

}  // namespace mixk

using namespace mixk;

// Sequences [0, num_decode) have one row each (step kernel); the others are portions.
extern "C" int mixk_retention(float* out, float* state, const void* q, int64_t q_stride,
                              const void* k, int64_t k_stride, const void* v, int64_t v_stride,
                              const float* powers, int n_powers, const float* cos_sin, int n_freq,
                              const int* positions, const int* seq_qstart, const int* seq_slot,
                              int S, int num_decode, int H, int dk, int dv, int dtype,
                              hipStream_t st) {
  if (S <= 0) return 0;
  if (dk <= 0 || dk > 256 || dv <= 0 || H <= 0 || n_powers != kChunk + 1 || 2 * n_freq > dk ||
      num_decode < 0 || num_decode > S)
    return -1;
  RetArgs a{out, state, q, k, v, powers, cos_sin, positions, seq_qstart, seq_slot, q_stride, k_stride,
            v_stride, H, dk, dv, n_freq, 0, 1.0f / sqrtf(static_cast<float>(dk))};
  const bool v4 = dv % 4 == 0 && (reinterpret_cast<uintptr_t>(state) & 15) == 0;
  const uintptr_t mask = dtype == 2 ? 31 : 15;
  const bool vec = dk % 16 == 0 && dv % 8 == 0 && n_freq % 8 == 0 && q_stride % 8 == 0 &&
                   k_stride % 8 == 0 && v_stride % 8 == 0 &&
                   ((reinterpret_cast<uintptr_t>(q) | reinterpret_cast<uintptr_t>(k) |
                     reinterpret_cast<uintptr_t>(v)) & mask) == 0 &&
                   (reinterpret_cast<uintptr_t>(cos_sin) & 31) == 0;
  int rc = 0;
  // portions longer than one row, or all sequences where the key is too wide for the chunk kernel
  const int steps = dk <= 128 ? num_decode : S;
  if (steps > 0) {
    MIXK_DISPATCH(dtype, rc = v4 ? (launch_step<T, true>(a, steps, st))
                                 : (launch_step<T, false>(a, steps, st)));
    if (rc) return rc;
  }
  if (steps < S) {
    a.seq0 = steps;
    const int seqs = S - steps;
#define MIXK_CHUNK(VEC)                                                                            \
  (dk <= 32 ? launch_chunk<T, 32, VEC>(a, seqs, st)                                                \
            : dk <= 64 ? launch_chunk<T, 64, VEC>(a, seqs, st) : launch_chunk<T, 128, VEC>(a, seqs, st))
    MIXK_DISPATCH(dtype, rc = vec ? MIXK_CHUNK(true) : MIXK_CHUNK(false));
#undef MIXK_CHUNK
  }
  return rc;
}
