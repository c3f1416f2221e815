// Causal paged attention whose weights are element-wise sigmoids mixed across the heads:
//     w_g(i, j) = sigmoid(cap tanh(scale q_g(i) . k(j) / cap) + bias[g])        (cap 0: no cap)
//     o_h(i)    = sum_j (sum_g talk[h, g] w_g(i, j)) v_h(j)
// for every j <= i, not normalised over the keys; k, v of a head are those of its KV head.  The
// mix needs every head's weight of a (query, key) pair before any head's values can be summed,
// so a workgroup owns all heads of its query rows.  Without a softmax there is no running
// maximum: partial sums over key ranges simply add up.  K pages are [nb, G, BS, dim], V pages
// channel-major [nb, G, vdim, BS].  Scores, weights and the mix are fp32 (see below).
//
// * matrix-core prefill kernel (bf16, dim % 8 == 0, vdim % 16 == 0, both <= 128, H <= 32): eight
//   waves, 16 query tokens, 32-key tiles; wave w owns HW = ceil(H / 8) consecutive heads, whose
//   Q fragments and O^T accumulators stay in its registers.  A head sits in slot
//   SL (h / HW) + h % HW of 8 SL slots (SL = 2 up to 16 heads, else 4), so a wave's heads are always
//   one run and any H is one K = 16 or 32 step of the mixing product.  Per tile:
//     A  S^T[16 keys x 16 tokens] = K . Q^T (mfma 16x16x32, K rows straight from the pages), the
//        weights in fp32, stored to LDS as an exact-to-2^-17 pair of bf16 (high + low part) in a
//        [key][token][slot] image;
//     B  mixed[16 keys x 16 heads] = W[16 keys x slots] . talk^T per token (two products, high
//        and low part, fp32 accumulation; talk holds bf16 checkpoint values), stored as bf16
//        [slot][token][key];
//     C  O^T[16 channels x 16 tokens] += V^T . mixed^T (V^T rows straight from the pages).
//   B needs A of all waves and C needs B of all waves; C of a tile and A of the next share one
//   barrier interval, so a tile costs two barriers (which order LDS only: the V fragments of the
//   tile are in flight during B, the first K fragments of the next one late in C).  The LDS images
//   are XOR-swizzled (sg_place) to spread the accesses of every phase over the banks.
//   A launch with few query tiles is split over the keys: every share writes fp32 partial rows, a
//   join kernel adds them.
// * matrix-core decode kernel (bf16, dim % 8 == 0, dim <= 256, vdim % 16 == 0, H <= 64): one
//   workgroup per (sequence, 64-key partition), columns = the query heads of a KV head; the mix
//   runs on the VALU in fp32; the partition's sums go to `part`, a combine kernel adds them.
// * rows kernel (any dtype and widths): fp32 FMA, all heads of up to 8 query rows per workgroup;
//   also the decode form of the shapes the matrix-core decode kernel does not take.
#include "mix_common.h"
#include "mixers.h"

namespace mixk {

typedef __attribute__((ext_vector_type(8))) __bf16 sg_bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 sg_bf16x4;
typedef __attribute__((ext_vector_type(4))) float sg_f32x4;
typedef __attribute__((ext_vector_type(4))) unsigned int sg_u32x4;

constexpr int kSgTile = 64;     // query tokens per entry of the host's tile list
constexpr int kSgTok = 16;      // query tokens per workgroup (matrix-core prefill)
constexpr int kSgKeys = 32;     // keys per tile
constexpr int kSgPart = 64;     // keys per decode partition
constexpr int kSgRow = kSgTok * 32;   // LDS row of a slot: 16 tokens x 32 keys
// head slots per wave (a run of 2 or 4, so 16 or 32 slots: the K of the mixing product)
__host__ __device__ constexpr int sg_slots(int HW) { return HW <= 2 ? 2 : 4; }
constexpr int kSgAcc = 64;      // accumulators per thread of the rows kernel
// heads per wave whose Q fragments live in LDS: the widest form is short of registers (it uses
// all of a CU's 160 KB)
__host__ __device__ constexpr int sg_q_lds(int HW, int ND) { return HW == 4 && ND == 4 ? 2 : 0; }
constexpr float kLog2e = 1.44269504088896341f;

struct SigArgs {
  const int* block_tables;
  const int* seq_kvlen;
  const int* seq_qstart;
  const int* tile_seq;
  const int* tile_qoff;
  float* part;          // decode partials [S, H, max_parts, vdim]
  const float* bias;    // [H]
  const float* talk;    // [H, H]
  int bt_width, H, G, dim, vdim, block_size, bs_shift, max_parts, rows;
  float scale, cap;
  float* split_out;     // prefill split over the keys: fp32 partial rows [split, T, H, vdim]
  int split, total_rows;
};

// Weight of one key on the fast transcendental units.  With a cap: t = tanh(y) as
// 1 - 2 / (1 + exp(2 y)); everything in log2 units with the constants folded by the caller:
//   k1 = 2 log2(e) scale / cap, k2 = 2 cap log2(e), k3 = -(cap + bias) log2(e)
// Without: k1 = -scale log2(e), k3 = -bias log2(e).
template <bool CAP>
__device__ __forceinline__ float sig_weight(float s, float k1, float k2, float k3) {
  float a;
  if (CAP) {
    const float r = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(s * k1));
    a = fmaf(k2, r, k3);
  } else {
    a = fmaf(s, k1, k3);
  }
  return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(a));
}

__device__ __forceinline__ sg_bf16x8 ld_frag(const __bf16* p) {
  return *reinterpret_cast<const sg_bf16x8*>(p);
}
__device__ __forceinline__ sg_bf16x8 zero_frag() {
  const sg_u32x4 z = {0u, 0u, 0u, 0u};
  return __builtin_bit_cast(sg_bf16x8, z);
}
// Place of (row, token, chunk) in an LDS image of rows of 16 tokens x 4 chunks of CH elements.  The
// token is XORed with the row and the chunk with the token's place, so that neither 16 tokens of a
// row nor 16 rows of a token share a bank.
template <int CH>
__device__ __forceinline__ int sg_place(int row, int t, int chunk) {
  const int p = t ^ (row & 15);
  return row * (kSgTok * 4 * CH) + p * (4 * CH) + (chunk ^ (p >> 2)) * CH;
}

// A copy the compiler knows nothing about: what is computed from it stays inside the loop instead of
// being hoisted into registers that the accumulators need.
__device__ __forceinline__ int fresh(int v) {
  asm volatile("" : "+v"(v));
  return v;
}

// Keys at or past kend of the 8 that start at t8 become zero (stale cache contents).
__device__ __forceinline__ sg_bf16x8 keep_keys(sg_bf16x8 v, int t8, int kend) {
#pragma unroll
  for (int j = 0; j < 8; ++j)
    if (t8 + j >= kend) v[j] = static_cast<__bf16>(0.f);
  return v;
}
// Workgroup barrier that orders LDS only: global loads in flight stay in flight.
__device__ __forceinline__ void lds_barrier() {
  __builtin_amdgcn_sched_barrier(0);
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  __builtin_amdgcn_sched_barrier(0);
}

// ONE: the heads of a wave share one KV head (H / G is a multiple of HW), so its K and V fragments
// are loaded once per tile, ahead of their use.
// Forms with few heads fit twice on a CU.
constexpr int sg_waves(int HW, int NV) { return HW * NV <= 8 ? 4 : 2; }

// V fragments in flight: what the registers leave.
constexpr int sg_v_flight(int HW, int NV) {
  return HW * NV >= 32 ? NV / 4 : (HW * NV == 8 && NV == 8 ? NV / 2 : NV);
}

template <int HW, int ND, int NV, bool CAP, bool ONE>   // dim <= 32 ND, vdim <= 16 NV, H <= 8 HW
__global__ void __launch_bounds__(512, sg_waves(HW, NV))
sigmoid_attention_mfma_kernel(__bf16* __restrict__ out, const __bf16* __restrict__ q,
                              const __bf16* __restrict__ k_cache,
                              const __bf16* __restrict__ v_cache, SigArgs a) {
  constexpr int QL = sg_q_lds(HW, ND), QR = HW - QL;     // heads with Q in LDS / in registers
  constexpr int QS = 32 * ND;                            // LDS row of one token's Q
  constexpr int NF = sg_v_flight(HW, NV);
  extern __shared__ __attribute__((aligned(16))) char sg_smem[];
  constexpr int SL = sg_slots(HW), kSlots = 8 * SL, CH = 2 * SL;   // CH: slots per chunk
  typedef __attribute__((ext_vector_type(SL))) __bf16 slots_t;           // a wave's slots
  typedef __attribute__((ext_vector_type(CH))) __bf16 chunk_t;           // K fragment of the mix
  __bf16* w_hi = reinterpret_cast<__bf16*>(sg_smem);     // [32 keys][16 tokens][kSlots]
  __bf16* w_lo = w_hi + kSgKeys * kSgTok * kSlots;
  __bf16* mixed = w_lo + kSgKeys * kSgTok * kSlots;      // [kSlots][16 tokens][32 keys]
  const int H = a.H, G = a.G, dim = a.dim, vdim = a.vdim, bs = a.block_size;
  const int rep = H / G, nv = vdim >> 4;
  // the tiles with the most keys come last in the list: start those first
  const int item = static_cast<int>(gridDim.x) - 1 - static_cast<int>(blockIdx.x);
  const int tile = item >> 2;
  const int s = a.tile_seq[tile], qo = a.tile_qoff[tile] + kSgTok * (item & 3);
  const int row0 = a.seq_qstart[s], n = a.seq_qstart[s + 1] - row0, kvlen = a.seq_kvlen[s];
  if (n <= 0 || kvlen <= 0 || qo >= n) return;
  const int ntok = min(kSgTok, n - qo);
  const int pos0 = kvlen - n + qo;          // position of the first query token
  const int kend = pos0 + ntok;             // keys [0, kend) are visible to somebody
  // this workgroup's share of the key tiles
  const int ntiles = (kend + kSgKeys - 1) / kSgKeys, per = (ntiles + a.split - 1) / a.split;
  const int kfirst = static_cast<int>(blockIdx.y) * per * kSgKeys;
  const int kstop = min(kend, kfirst + per * kSgKeys);
  const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, c = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h0 = w * HW;
  const bool wave_on = h0 < H;
  const int qpos = pos0 + r;
  // head QR + e of the wave in LDS: this lane's row of the e-th 16-token block, chunks XORed with r
  __bf16* q_rows = mixed + kSlots * kSgRow + (w * QL * kSgTok + r) * QS;
  auto q_lds = [&](int e, int st, int rr) {
    return q_rows + e * kSgTok * QS + (((st * 4 + c) ^ (rr & (4 * ND - 1))) << 3);
  };

  // Q fragments; channels past dim, tokens past ntok and heads past H are zero
  sg_bf16x8 qf[QR > 0 ? QR : 1][ND];
  float k3[HW];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int h = h0 + hh;
    // a head past H: exp2(inf) makes every weight an exact zero
    k3[hh] = h < H ? -((CAP ? a.cap : 0.f) + a.bias[h]) * kLog2e : INFINITY;
#pragma unroll
    for (int st = 0; st < ND; ++st) {
      sg_bf16x8 f = zero_frag();
      if (r < ntok && h < H && st * 32 + 8 * c < dim)
        f = ld_frag(q + (static_cast<int64_t>(row0 + qo + r) * H + h) * dim + st * 32 + 8 * c);
      if (hh < QR)
        qf[hh < QR ? hh : 0][st] = f;
      else
        *reinterpret_cast<sg_bf16x8*>(q_lds(hh - QR, st, r)) = f;   // read back by this lane only
    }
  }
  const float k1 = CAP ? 2.0f * kLog2e * a.scale / a.cap : -kLog2e * a.scale;
  const float k2 = 2.0f * a.cap * kLog2e;
  // B operand of the mix: column = output slot, rows = this lane's CH input slots
  chunk_t tf[kSlots / 16];
#pragma unroll
  for (int ht = 0; ht < kSlots / 16; ++ht) {
    const int so = ht * 16 + r;
    const int ho = (so / SL) * HW + so % SL;
#pragma unroll
    for (int j = 0; j < CH; ++j) {
      const int si = CH * c + j;
      const int hi = (si / SL) * HW + si % SL;
      const bool ok = so % SL < HW && ho < H && si % SL < HW && hi < H;
      tf[ht][j] = static_cast<__bf16>(ok ? a.talk[ho * H + hi] : 0.f);
    }
  }
  const int nht = ((H - 1) / HW * SL + HW + 15) / 16;   // output slot tiles in use
  auto mix = [](chunk_t x, chunk_t t, sg_f32x4 d) {
    if constexpr (SL == 4) {
      return __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, t, d, 0, 0, 0);
    } else {
      typedef __attribute__((ext_vector_type(4))) short s16x4;
      return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(s16x4, x),
                                                       __builtin_bit_cast(s16x4, t), d, 0, 0, 0);
    }
  };
  sg_f32x4 O[HW][NV];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh)
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) O[hh][vt] = sg_f32x4{0.f, 0.f, 0.f, 0.f};

  // Addresses are clamped instead of predicated: a key past the end reads the last key (its
  // weight is masked), a channel group past dim reads group 0 (its Q is zero), a channel tile
  // past vdim reads the last one (never stored), a head past H the last one (zero weights).
  const int* bt = a.block_tables + static_cast<int64_t>(s) * a.bt_width;
  const int64_t kpage = static_cast<int64_t>(G) * bs * dim, vpage = static_cast<int64_t>(G) * vdim * bs;
  const int shift = a.bs_shift, bmask = bs - 1, last = kend - 1;
  auto kv_head = [&](int hh) { return min(h0 + hh, H - 1) / rep; };
  auto page_at = [&](int key) { return bt[min(key, last) >> shift]; };
  const int g0 = kv_head(0);
  int koff[ND];
#pragma unroll
  for (int st = 0; st < ND; ++st) koff[st] = st * 32 + 8 * c < dim ? st * 32 + 8 * c : 0;

  auto load_k = [&](sg_bf16x8 (&kf)[ND], int page, int key, int g) {
    const __bf16* kb = k_cache + page * kpage +
                       static_cast<int64_t>(g * bs + (min(key, last) & bmask)) * dim;
#pragma unroll
    for (int st = 0; st < ND; ++st) kf[st] = ld_frag(kb + koff[st]);
  };
  auto head_scores = [&](const sg_bf16x8 (&kf)[ND], int hh, int rr) {
    sg_f32x4 S = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < ND; ++st) {
      const sg_bf16x8 f = hh < QR ? qf[hh < QR ? hh : 0][st] : ld_frag(q_lds(hh - QR, st, rr));
      S = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[st], f, S, 0, 0, 0);
    }
    return S;
  };
  // weights of keys k0 + 16 sub .. + 15 for the wave's heads, into the LDS image
  auto weights = [&](int k0, int sub, const sg_f32x4 (&S)[HW]) {
    const int kb = k0 + sub * 16 + 4 * c;
    const bool edge = k0 + kSgKeys - 1 > pos0;   // some key lies after the first query token
    const int rr = fresh(r);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      slots_t hi, lo;
#pragma unroll
      for (int hh = 0; hh < SL; ++hh) {
        float x = 0.f;
        if (hh < HW) {
          x = sig_weight<CAP>(S[hh < HW ? hh : 0][i], k1, k2, k3[hh < HW ? hh : 0]);
          if (edge && kb + i > qpos) x = 0.f;
        }
        hi[hh] = static_cast<__bf16>(x);
        lo[hh] = static_cast<__bf16>(x - static_cast<float>(hi[hh]));
      }
      const int o = sg_place<CH>(sub * 16 + 4 * c + i, rr, w >> 1) + (w & 1) * SL;
      *reinterpret_cast<slots_t*>(w_hi + o) = hi;
      *reinterpret_cast<slots_t*>(w_lo + o) = lo;
    }
  };

  sg_bf16x8 ka[ND];   // ONE: K of the next tile's first 16 keys, in flight
  auto scores = [&](int k0, int pg0, int pg1) {
    const int rr = fresh(r);
    if (ONE) {
      sg_bf16x8 kb[ND];
      sg_f32x4 S[HW];
#pragma unroll
      for (int hh = 0; hh < HW; ++hh) S[hh] = head_scores(ka, hh, rr);
      // the second half's K loads take over the first half's registers and land during its weights
      __builtin_amdgcn_sched_barrier(0);
      load_k(kb, pg1, k0 + 16 + r, g0);
      __builtin_amdgcn_sched_barrier(0);
      weights(k0, 0, S);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int hh = 0; hh < HW; ++hh) S[hh] = head_scores(kb, hh, rr);
      weights(k0, 1, S);
    } else {
#pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
        sg_f32x4 S[HW];
#pragma unroll
        for (int hh = 0; hh < HW; ++hh) {
          sg_bf16x8 kf[ND];
          load_k(kf, sub ? pg1 : pg0, k0 + sub * 16 + r, kv_head(hh));
          S[hh] = head_scores(kf, hh, rr);
        }
        weights(k0, sub, S);
      }
    }
  };

  // (a share without keys runs the prologue on clamped addresses and stores zeros)
  int pk0 = page_at(kfirst + r), pk1 = page_at(kfirst + 16 + r), pv = page_at(kfirst + 8 * c);
  if (wave_on) {
    if (ONE) load_k(ka, pk0, kfirst + r, g0);
    scores(kfirst, pk0, pk1);
  } else {   // this wave's slots never hold a head: zero them once
    slots_t z;
#pragma unroll
    for (int hh = 0; hh < SL; ++hh) z[hh] = static_cast<__bf16>(0.f);
    for (int key = c; key < kSgKeys; key += 4) {
      const int o = sg_place<CH>(key, r, w >> 1) + (w & 1) * SL;
      *reinterpret_cast<slots_t*>(w_hi + o) = z;
      *reinterpret_cast<slots_t*>(w_lo + o) = z;
    }
  }
  pk0 = page_at(kfirst + kSgKeys + r);
  pk1 = page_at(kfirst + kSgKeys + 16 + r);
  for (int k0 = kfirst; k0 < kstop; k0 += kSgKeys) {
    const int nk = k0 + kSgKeys, t8 = k0 + 8 * c;
    const __bf16* vb = v_cache + pv * vpage + (min(t8, last) & bmask & ~7) + static_cast<int64_t>(r) * bs;
    sg_bf16x8 vf[NF];
    auto load_v = [&](int vt0) {
#pragma unroll
      for (int e = 0; e < NF; ++e)
        vf[e] = ld_frag(vb + static_cast<int64_t>(g0 * vdim + min(vt0 + e, nv - 1) * 16) * bs);
    };
    if (ONE && wave_on) load_v(0);
    pv = page_at(nk + 8 * c);
    lds_barrier();
    const int rb = fresh(r);
    // B: the wave mixes the pairs of tokens 2 w and 2 w + 1
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      const int t = 2 * w + tt;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int o = sg_place<CH>(half * 16 + rb, t, c);
        const chunk_t ah = *reinterpret_cast<const chunk_t*>(w_hi + o);
        const chunk_t al = *reinterpret_cast<const chunk_t*>(w_lo + o);
#pragma unroll
        for (int ht = 0; ht < kSlots / 16; ++ht) {
          if (ht < nht) {
            sg_f32x4 D = {0.f, 0.f, 0.f, 0.f};
            D = mix(al, tf[ht], D);
            D = mix(ah, tf[ht], D);
            sg_bf16x4 e;
#pragma unroll
            for (int i = 0; i < 4; ++i) e[i] = static_cast<__bf16>(D[i]);
            *reinterpret_cast<sg_bf16x4*>(mixed + sg_place<8>(ht * 16 + rb, t, half * 2 + (c >> 1)) +
                                          (c & 1) * 4) = e;
          }
        }
      }
    }
    lds_barrier();
    if (wave_on) {   // C
      const bool tail = nk > kend;
      const int rc = fresh(r);
      if (ONE) {
#pragma unroll
        for (int vt0 = 0; vt0 < NV; vt0 += NF) {
          if (vt0 > 0) load_v(vt0);
          if (vt0 + NF >= NV && NF < NV) load_k(ka, pk0, nk + r, g0);
          if (tail) {
#pragma unroll
            for (int e = 0; e < NF; ++e) vf[e] = keep_keys(vf[e], t8, kend);
          }
#pragma unroll
          for (int hh = 0; hh < HW; ++hh) {
            const sg_bf16x8 pf = ld_frag(mixed + sg_place<8>(SL * w + hh, rc, c));
#pragma unroll
            for (int e = 0; e < NF; ++e)
              O[hh][vt0 + e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[e], pf, O[hh][vt0 + e], 0, 0, 0);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
        if (NF == NV) load_k(ka, pk0, nk + r, g0);
        __builtin_amdgcn_sched_barrier(0);
      } else {
#pragma unroll
        for (int hh = 0; hh < HW; ++hh) {
          const sg_bf16x8 pf = ld_frag(mixed + sg_place<8>(SL * w + hh, rc, c));
          const __bf16* vh = vb + static_cast<int64_t>(kv_head(hh)) * vdim * bs;
          sg_bf16x8 vg[NV];
#pragma unroll
          for (int vt = 0; vt < NV; ++vt)
            vg[vt] = ld_frag(vh + static_cast<int64_t>(min(vt, nv - 1)) * 16 * bs);
          if (tail) {
#pragma unroll
            for (int vt = 0; vt < NV; ++vt) vg[vt] = keep_keys(vg[vt], t8, kend);
          }
#pragma unroll
          for (int vt = 0; vt < NV; ++vt)
            O[hh][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vg[vt], pf, O[hh][vt], 0, 0, 0);
        }
      }
      if (nk < kstop) scores(nk, pk0, pk1);
    }
    pk0 = page_at(nk + kSgKeys + r);
    pk1 = page_at(nk + kSgKeys + 16 + r);
  }
  if (!wave_on || r >= ntok) return;
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int h = h0 + hh;
    if (h < H) {
      if (a.split > 1) {
        const int64_t row = static_cast<int64_t>(blockIdx.y) * a.total_rows + row0 + qo + r;
        float* o = a.split_out + (row * H + h) * vdim + 4 * c;
#pragma unroll
        for (int vt = 0; vt < NV; ++vt)
          if (vt < nv) *reinterpret_cast<sg_f32x4*>(o + vt * 16) = O[hh][vt];
        continue;
      }
      __bf16* o = out + (static_cast<int64_t>(row0 + qo + r) * H + h) * vdim + 4 * c;
#pragma unroll
      for (int vt = 0; vt < NV; ++vt) {
        if (vt < nv) {
          sg_bf16x4 e;
#pragma unroll
          for (int i = 0; i < 4; ++i) e[i] = static_cast<__bf16>(O[hh][vt][i]);
          *reinterpret_cast<sg_bf16x4*>(o + vt * 16) = e;
        }
      }
    }
  }
}

// Rows of the tile list: the sum of the key shares' partial rows.
__global__ void sigmoid_attention_join_kernel(__bf16* __restrict__ out, SigArgs a) {
  const int s = a.tile_seq[blockIdx.x], qo = a.tile_qoff[blockIdx.x] + blockIdx.y;
  const int row0 = a.seq_qstart[s], n = a.seq_qstart[s + 1] - row0;
  if (qo >= n || a.seq_kvlen[s] <= 0) return;
  const int width = a.H * a.vdim;   // a multiple of 16
  const int64_t base = static_cast<int64_t>(row0 + qo) * width;
  for (int i = threadIdx.x * 8; i < width; i += blockDim.x * 8) {
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int z = 0; z < a.split; ++z) {
      float p[8];
      ld8(a.split_out + static_cast<int64_t>(z) * a.total_rows * width + base + i, p);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] += p[e];
    }
    st8(out + base + i, v);
  }
}

// One workgroup of eight waves per (decode sequence, 64-key partition), all heads.
constexpr int kSgMixRow = kSgPart + 8;
// dynamic LDS: mixed weights bf16 [H][72], weights fp32 [64 keys][H + 1], talk fp32 [H][H]
__host__ __device__ constexpr size_t sg_decode_smem(int H) {
  return sizeof(__bf16) * H * kSgMixRow + sizeof(float) * (kSgPart * (H + 1) + H * H);
}

template <int ND, bool CAP>   // dim <= 32 ND
__global__ void __launch_bounds__(512)
sigmoid_attention_decode_kernel(const __bf16* __restrict__ q, const __bf16* __restrict__ k_cache,
                                const __bf16* __restrict__ v_cache, SigArgs a) {
  extern __shared__ __attribute__((aligned(16))) char sg_smem[];
  const int H = a.H, G = a.G, dim = a.dim, vdim = a.vdim, bs = a.block_size, HS = H + 1;
  constexpr int PR = kSgMixRow;
  __bf16* mixed = reinterpret_cast<__bf16*>(sg_smem);
  float* wts = reinterpret_cast<float*>(sg_smem + sizeof(__bf16) * H * PR);
  float* talk = wts + kSgPart * HS;
  const int s = blockIdx.x, kbeg = blockIdx.y * kSgPart;
  const int kvlen = a.seq_kvlen[s];
  const int kend = min(kvlen, kbeg + kSgPart);
  if (kbeg >= kend) return;
  const int rep = H / G, ct = (rep + 15) >> 4, last = kend - 1;
  const int lane = threadIdx.x & 63, r = lane & 15, c = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(static_cast<int>(threadIdx.x) >> 6);
  const int* bt = a.block_tables + static_cast<int64_t>(s) * a.bt_width;
  const int64_t row = a.seq_qstart[s];
  const float k1 = CAP ? 2.0f * kLog2e * a.scale / a.cap : -kLog2e * a.scale;
  const float k2 = 2.0f * a.cap * kLog2e;
  const int shift = a.bs_shift, bmask = bs - 1;
  // the V pages of this lane's key groups (clamped like every address here)
  const __bf16* vb[2];
#pragma unroll
  for (int ks = 0; ks < 2; ++ks) {
    const int t8 = min(kbeg + ks * 32 + 8 * c, last);
    vb[ks] = v_cache + static_cast<int64_t>(bt[t8 >> shift]) * G * vdim * bs + (t8 & bmask & ~7) +
             static_cast<int64_t>(r) * bs;
  }
  for (int i = threadIdx.x; i < H * H; i += 512) talk[i] = a.talk[i];
  // waves w and w + 4 score keys 16 (w & 3) .. + 15 of the partition, every other KV head each
  {
    const int key = min(kbeg + 16 * (w & 3) + r, last);
    const __bf16* kb = k_cache + static_cast<int64_t>(bt[key >> shift]) * G * bs * dim +
                       static_cast<int64_t>(key & bmask) * dim;
#pragma unroll 2
    for (int j = w >> 2; j < G * ct; j += 2) {
      const int g = j / ct, hl = (j - g * ct) * 16 + r, h = g * rep + hl;
      const bool hok = hl < rep;
      const __bf16* qr = q + (row * H + min(h, H - 1)) * dim;
      sg_bf16x8 kf[ND], qf[ND];
#pragma unroll
      for (int st = 0; st < ND; ++st) {
        const int ch = st * 32 + 8 * c;
        kf[st] = ld_frag(kb + static_cast<int64_t>(g) * bs * dim + (ch < dim ? ch : 0));
        qf[st] = ch < dim ? ld_frag(qr + ch) : zero_frag();
      }
      const float k3 = -((CAP ? a.cap : 0.f) + a.bias[min(h, H - 1)]) * kLog2e;
      sg_f32x4 S = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < ND; ++st)
        S = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[st], qf[st], S, 0, 0, 0);
      if (hok) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int kk = 16 * (w & 3) + 4 * c + i;
          wts[kk * HS + h] = kbeg + kk < kend ? sig_weight<CAP>(S[i], k1, k2, k3) : 0.f;
        }
      }
    }
  }
  __syncthreads();
  // lane = key, four output heads per pass of a wave
  for (int hb = 4 * w; hb < H; hb += 32) {
    float m[4] = {0.f, 0.f, 0.f, 0.f};
    const float* tr[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) tr[e] = talk + min(hb + e, H - 1) * H;
#pragma unroll 4
    for (int g = 0; g < H; ++g) {
      const float x = wts[lane * HS + g];
#pragma unroll
      for (int e = 0; e < 4; ++e) m[e] = fmaf(tr[e][g], x, m[e]);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (hb + e < H) mixed[(hb + e) * PR + lane] = static_cast<__bf16>(m[e]);
  }
  __syncthreads();
  const int nv = vdim >> 4;
#pragma unroll 4
  for (int j = w; j < G * ct * nv; j += 8) {
    const int vt = j % nv, gc = j / nv;
    const int g = gc / ct, hl = (gc - g * ct) * 16 + r, h = g * rep + hl;
    const int64_t vo = static_cast<int64_t>(g * vdim + vt * 16) * bs;
    sg_bf16x8 vf[2], pf[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      vf[ks] = ld_frag(vb[ks] + vo);
      pf[ks] = hl < rep ? ld_frag(mixed + h * PR + ks * 32 + 8 * c) : zero_frag();
    }
    sg_f32x4 O = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks)
      O = __builtin_amdgcn_mfma_f32_16x16x32_bf16(keep_keys(vf[ks], kbeg + ks * 32 + 8 * c, kend),
                                                  pf[ks], O, 0, 0, 0);
    if (hl < rep)
      *reinterpret_cast<sg_f32x4*>(a.part + ((static_cast<int64_t>(s) * H + h) * a.max_parts +
                                             blockIdx.y) * vdim + vt * 16 + 4 * c) = O;
  }
}

// Sum of the partitions of one (decode sequence, head).
template <typename T>
__global__ void sigmoid_attention_combine_kernel(T* __restrict__ out, SigArgs a) {
  const int s = blockIdx.x, h = blockIdx.y, vdim = a.vdim;
  const int kvlen = a.seq_kvlen[s];
  if (kvlen <= 0) return;
  const int np = min(a.max_parts, (kvlen + kSgPart - 1) / kSgPart);
  const float* base = a.part + (static_cast<int64_t>(s) * a.H + h) * a.max_parts * vdim;
  T* o = out + (static_cast<int64_t>(a.seq_qstart[s]) * a.H + h) * vdim;
  for (int d = threadIdx.x; d < vdim; d += blockDim.x) {
    float v = 0.f;
#pragma unroll 8
    for (int p = 0; p < np; ++p) v += base[static_cast<int64_t>(p) * vdim + d];
    stf(o + d, v);
  }
}

// All heads of `rows` query rows (a divisor of 64; 1 in decode, over one partition of the keys).
template <typename T, bool DECODE>
__global__ void __launch_bounds__(256)
sigmoid_attention_rows_kernel(T* __restrict__ out, const T* __restrict__ q,
                              const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                              SigArgs a) {
  extern __shared__ __attribute__((aligned(16))) char sg_smem[];
  const int H = a.H, G = a.G, dim = a.dim, vdim = a.vdim, bs = a.block_size, rep = H / G;
  const int R = DECODE ? 1 : a.rows;
  int s, qo, n, kbeg, kend, kvlen, row0, nrows;
  if (DECODE) {
    s = blockIdx.x;
    qo = 0;
    n = nrows = 1;
    row0 = a.seq_qstart[s];
    kvlen = a.seq_kvlen[s];
    kbeg = blockIdx.y * kSgPart;
    kend = min(kvlen, kbeg + kSgPart);
    if (kbeg >= kend) return;
  } else {
    const int per = kSgTile / R, tile = blockIdx.x / per;
    s = a.tile_seq[tile];
    qo = a.tile_qoff[tile] + R * (blockIdx.x - tile * per);
    row0 = a.seq_qstart[s];
    n = a.seq_qstart[s + 1] - row0;
    kvlen = a.seq_kvlen[s];
    if (n <= 0 || kvlen <= 0 || qo >= n) return;
    nrows = min(R, n - qo);
    kbeg = 0;
    kend = kvlen - n + qo + nrows;
  }
  float* qs = reinterpret_cast<float*>(sg_smem);   // [R * H][dim]
  float* ws = qs + R * H * dim;                    // [R * H][32] weights
  float* ms = ws + R * H * kSgKeys;                // [R * H][32] mixed weights
  const int tid = threadIdx.x, items = nrows * H;
  for (int i = tid; i < items * dim; i += 256)
    qs[i] = ldf(q + static_cast<int64_t>(row0 + qo) * H * dim + i);
  float acc[kSgAcc];
#pragma unroll
  for (int j = 0; j < kSgAcc; ++j) acc[j] = 0.f;
  const int* bt = a.block_tables + static_cast<int64_t>(s) * a.bt_width;
  __syncthreads();
  for (int k0 = kbeg; k0 < kend; k0 += kSgKeys) {
    for (int i = tid; i < items * kSgKeys; i += 256) {
      const int kk = i & (kSgKeys - 1), rh = i >> 5, rr = rh / H, h = rh - rr * H;
      const int key = k0 + kk, qpos = kvlen - n + qo + rr;
      float x = 0.f;
      if (key < kend && key <= qpos) {
        const T* kr = k_cache + ((static_cast<int64_t>(bt[key / bs]) * G + h / rep) * bs + key % bs) * dim;
        const float* qr = qs + rh * dim;
        float dot = 0.f;
        for (int d = 0; d < dim; ++d) dot += qr[d] * ldf(kr + d);
        float z = dot * a.scale;
        if (a.cap > 0.f) z = a.cap * tanhf(z / a.cap);
        x = sigmoidf_(z + a.bias[h]);
      }
      ws[i] = x;
    }
    __syncthreads();
    for (int i = tid; i < items * kSgKeys; i += 256) {
      const int kk = i & (kSgKeys - 1), rh = i >> 5, rr = rh / H, h = rh - rr * H;
      const float* wr = ws + rr * H * kSgKeys + kk;
      const float* tr = a.talk + static_cast<int64_t>(h) * H;
      float m = 0.f;
      for (int g = 0; g < H; ++g) m = fmaf(tr[g], wr[g * kSgKeys], m);
      ms[i] = m;
    }
    __syncthreads();
    const int kn = min(kSgKeys, kend - k0);
#pragma unroll
    for (int j = 0; j < kSgAcc; ++j) {
      const int i = tid + 256 * j;
      if (i < items * vdim) {
        const int rh = i / vdim, v = i - rh * vdim, g = (rh % H) / rep;
        const float* mr = ms + rh * kSgKeys;
        float s_ = acc[j];
        for (int kk = 0; kk < kn; ++kk) {
          const int key = k0 + kk;
          s_ += mr[kk] * ldf(v_cache + ((static_cast<int64_t>(bt[key / bs]) * G + g) * vdim + v) * bs +
                             key % bs);
        }
        acc[j] = s_;
      }
    }
    // the next tile's weights go to ws, which nobody reads any more; ms is rewritten only after
    // the barrier that follows them
  }
#pragma unroll
  for (int j = 0; j < kSgAcc; ++j) {
    const int i = tid + 256 * j;
    if (i < items * vdim) {
      if (DECODE) {
        const int h = i / vdim, v = i - h * vdim;
        a.part[((static_cast<int64_t>(s) * H + h) * a.max_parts + blockIdx.y) * vdim + v] = acc[j];
      } else {
        stf(out + static_cast<int64_t>(row0 + qo) * H * vdim + i, acc[j]);
      }
    }
  }
}

template <typename K>
int sg_smem_opt_in(K kernel, size_t smem) {
  if (smem <= 48 * 1024) return 0;
  return static_cast<int>(hipFuncSetAttribute(reinterpret_cast<const void*>(kernel),
                                              hipFuncAttributeMaxDynamicSharedMemorySize,
                                              static_cast<int>(smem)));
}

template <int HW, int ND, int NV, bool CAP, bool ONE>
int sg_launch_prefill(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
                      int num_tiles, hipStream_t st) {
  constexpr size_t smem = sizeof(__bf16) * (3 * kSgKeys * kSgTok * 8 * sg_slots(HW) +
                                            sg_q_lds(HW, ND) * 8 * kSgTok * 32 * ND);
  static_assert(smem <= 160 * 1024, "LDS of a CU");
  static bool opted = false;
  if (!opted) {
    if (int rc = sg_smem_opt_in(sigmoid_attention_mfma_kernel<HW, ND, NV, CAP, ONE>, smem)) return rc;
    opted = true;
  }
  hipLaunchKernelGGL((sigmoid_attention_mfma_kernel<HW, ND, NV, CAP, ONE>),
                     dim3(num_tiles * (kSgTile / kSgTok), a.split), dim3(512), smem, st,
                     static_cast<__bf16*>(out), static_cast<const __bf16*>(q),
                     static_cast<const __bf16*>(k), static_cast<const __bf16*>(v), a);
  if (a.split > 1)
    hipLaunchKernelGGL(sigmoid_attention_join_kernel, dim3(num_tiles, kSgTile), dim3(256), 0, st,
                       static_cast<__bf16*>(out), a);
  return static_cast<int>(hipGetLastError());
}

template <int HW, int ND, int NV, bool CAP>
int sg_prefill_kv(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
                  int num_tiles, hipStream_t st) {
  if constexpr (HW > 1) {
    if ((a.H / a.G) % HW != 0)
      return sg_launch_prefill<HW, ND, NV, CAP, false>(out, q, k, v, a, num_tiles, st);
  }
  return sg_launch_prefill<HW, ND, NV, CAP, true>(out, q, k, v, a, num_tiles, st);
}

template <int HW, bool CAP>
int sg_prefill_dims(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
                    int num_tiles, hipStream_t st) {
  if (a.dim <= 64 && a.vdim <= 64) return sg_prefill_kv<HW, 2, 4, CAP>(out, q, k, v, a, num_tiles, st);
  return sg_prefill_kv<HW, 4, 8, CAP>(out, q, k, v, a, num_tiles, st);
}

template <bool CAP>
int sg_prefill(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
               int num_tiles, hipStream_t st) {
  switch ((a.H + 7) / 8) {
    case 1: return sg_prefill_dims<1, CAP>(out, q, k, v, a, num_tiles, st);
    case 2: return sg_prefill_dims<2, CAP>(out, q, k, v, a, num_tiles, st);
    case 3: return sg_prefill_dims<3, CAP>(out, q, k, v, a, num_tiles, st);
    default: return sg_prefill_dims<4, CAP>(out, q, k, v, a, num_tiles, st);
  }
}

template <int ND, bool CAP>
void sg_launch_decode(const void* q, const void* k, const void* v, const SigArgs& a,
                      int num_decode, int parts, hipStream_t st) {
  static_assert(sg_decode_smem(64) <= 48 * 1024, "no opt-in needed up to 64 heads");
  const size_t smem = sg_decode_smem(a.H);
  hipLaunchKernelGGL((sigmoid_attention_decode_kernel<ND, CAP>), dim3(num_decode, parts), dim3(512),
                     smem, st, static_cast<const __bf16*>(q), static_cast<const __bf16*>(k),
                     static_cast<const __bf16*>(v), a);
}

// dynamic LDS of the rows kernel at R rows
size_t sg_rows_smem(const SigArgs& a, int R) {
  return sizeof(float) * static_cast<size_t>(R) * a.H * (a.dim + 2 * kSgKeys);
}

template <typename T>
int sg_launch_rows(void* out, const void* q, const void* k, const void* v, SigArgs a,
                   int num_tiles, int num_decode, int parts, hipStream_t st) {
  int R = 8;
  while (R > 1 && (static_cast<int64_t>(R) * a.H * a.vdim > 256 * kSgAcc || sg_rows_smem(a, R) > 64 * 1024))
    R >>= 1;
  if (static_cast<int64_t>(R) * a.H * a.vdim > 256 * kSgAcc || sg_rows_smem(a, R) > 150 * 1024) return -1;
  a.rows = R;
  if (num_tiles > 0) {
    const size_t smem = sg_rows_smem(a, R);
    if (int rc = sg_smem_opt_in(sigmoid_attention_rows_kernel<T, false>, smem)) return rc;
    hipLaunchKernelGGL((sigmoid_attention_rows_kernel<T, false>), dim3(num_tiles * (kSgTile / R)),
                       dim3(256), smem, st, static_cast<T*>(out), static_cast<const T*>(q),
                       static_cast<const T*>(k), static_cast<const T*>(v), a);
  }
  if (num_decode > 0) {
    const size_t smem = sg_rows_smem(a, 1);
    if (int rc = sg_smem_opt_in(sigmoid_attention_rows_kernel<T, true>, smem)) return rc;
    hipLaunchKernelGGL((sigmoid_attention_rows_kernel<T, true>), dim3(num_decode, parts), dim3(256),
                       smem, st, static_cast<T*>(out), static_cast<const T*>(q),
                       static_cast<const T*>(k), static_cast<const T*>(v), a);
  }
  return static_cast<int>(hipGetLastError());
}

}  // namespace mixk

using namespace mixk;

// Prefill tiles of 64 query tokens (tile_seq / tile_qoff) and decode sequences [0, num_decode) (one
// query row each, row = seq_qstart[s]; partials in `part` [num_decode, H, max_parts, vdim] fp32,
// max_parts >= ceil(max_decode_kv / 64)).
extern "C" int mixk_sigmoid_attention(void* out, const void* q, const void* k_cache,
                                      const void* v_cache, const int* block_tables, int bt_width,
                                      const int* seq_kvlen, const int* seq_qstart,
                                      const int* tile_seq, const int* tile_qoff, int num_tiles,
                                      int num_decode, int max_decode_kv, float* part,
                                      int max_parts, int H, int G, int dim, int vdim,
                                      int block_size, float scale, float cap, const float* bias,
                                      const float* talk, float* split_out, int split,
                                      int total_rows, int use_mfma, int dtype, hipStream_t st) {
  if (num_tiles <= 0 && num_decode <= 0) return 0;
  if (G <= 0 || H % G != 0 || cap < 0.f || split < 1) return -1;
  const int parts = (max_decode_kv + kSgPart - 1) / kSgPart;
  if (num_decode > 0 && (parts < 1 || parts > max_parts || part == nullptr)) return -1;
  int bs_shift = 0;
  while ((1 << bs_shift) < block_size) ++bs_shift;
  const SigArgs a{block_tables, seq_kvlen, seq_qstart, tile_seq, tile_qoff, part, bias, talk,
                  bt_width, H, G, dim, vdim, block_size, bs_shift, max_parts, 0, scale, cap,
                  split_out, split_out != nullptr ? split : 1, total_rows};
  const bool pages_ok = block_size >= 8 && (block_size & (block_size - 1)) == 0;
  const bool base_ok = use_mfma && dtype == 0 && pages_ok && dim % 8 == 0 && vdim % 16 == 0;
  int rc = 0, rows_tiles = num_tiles, rows_decode = num_decode;
  if (num_tiles > 0 && base_ok && dim <= 128 && vdim <= 128 && H <= 32) {
    rc = cap > 0.f ? sg_prefill<true>(out, q, k_cache, v_cache, a, num_tiles, st)
                   : sg_prefill<false>(out, q, k_cache, v_cache, a, num_tiles, st);
    if (rc) return rc;
    rows_tiles = 0;
  }
  if (num_decode > 0 && base_ok && dim <= 256 && H <= 64) {
#define MIXK_SG_DECODE(ND)                                                               \
  (cap > 0.f ? sg_launch_decode<ND, true>(q, k_cache, v_cache, a, num_decode, parts, st) \
             : sg_launch_decode<ND, false>(q, k_cache, v_cache, a, num_decode, parts, st))
    if (dim <= 64)
      MIXK_SG_DECODE(2);
    else if (dim <= 128)
      MIXK_SG_DECODE(4);
    else
      MIXK_SG_DECODE(8);
#undef MIXK_SG_DECODE
    rc = static_cast<int>(hipGetLastError());
    if (rc) return rc;
    rows_decode = 0;
  }
  if (rows_tiles > 0 || rows_decode > 0) {
    MIXK_DISPATCH(dtype, rc = sg_launch_rows<T>(out, q, k_cache, v_cache, a, rows_tiles,
                                                rows_decode, parts, st));
    if (rc) return rc;
  }
  if (num_decode > 0)
    MIXK_DISPATCH(dtype, hipLaunchKernelGGL(sigmoid_attention_combine_kernel<T>,
                                            dim3(num_decode, H), dim3(kWave), 0, st,
                                            static_cast<T*>(out), a));
  return static_cast<int>(hipGetLastError());
}
