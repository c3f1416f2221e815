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
//   4 (h / HW) + h % HW of 32 slots, so a wave's heads are always one 8-byte run and any H <= 32
//   is one K = 32 step of the mixing product.  Per tile:
//     A  S^T[16 keys x 16 tokens] = K . Q^T (mfma 16x16x32, K rows straight from the pages), the
//        weights in fp32, stored to LDS as an exact-to-2^-17 pair of bf16 (high + low part) in a
//        [key][token][slot] image;
//     B  mixed[16 keys x 16 heads] = W[16 keys x 32 slots] . talk^T per token (two products, high
//        and low part, fp32 accumulation; talk holds bf16 checkpoint values), stored as bf16
//        [slot][token][key];
//     C  O^T[16 channels x 16 tokens] += V^T . mixed^T (V^T rows straight from the pages).
//   B needs A of all waves and C needs B of all waves; C of a tile and A of the next share one
//   barrier interval, so a tile costs two barriers.  Row strides and an XOR of the 16-byte chunk
//   with bits of the token keep the LDS accesses conflict-free.
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
constexpr int kSgSlots = 32;    // head slots
constexpr int kSgRow = kSgTok * 32 + 8;   // LDS row of 16 tokens x 32 bf16, padded by 16 bytes
constexpr int kSgAcc = 64;      // accumulators per thread of the rows kernel
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
// 8 keys of a V^T row starting at key t8; keys at or past kend become zero
__device__ __forceinline__ sg_bf16x8 ld_v(const __bf16* p, int t8, int kend) {
  if (t8 >= kend) return zero_frag();
  sg_bf16x8 v = ld_frag(p);
  if (t8 + 8 > kend) {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (t8 + j >= kend) v[j] = static_cast<__bf16>(0.f);
  }
  return v;
}

template <int HW, int ND, int NV, bool CAP>   // dim <= 32 ND, vdim <= 16 NV, H <= 8 HW
__global__ void __launch_bounds__(512)
sigmoid_attention_mfma_kernel(__bf16* __restrict__ out, const __bf16* __restrict__ q,
                              const __bf16* __restrict__ k_cache,
                              const __bf16* __restrict__ v_cache, SigArgs a) {
  extern __shared__ __attribute__((aligned(16))) char sg_smem[];
  __bf16* w_hi = reinterpret_cast<__bf16*>(sg_smem);     // [32 keys][kSgRow]
  __bf16* w_lo = w_hi + kSgKeys * kSgRow;
  __bf16* mixed = w_lo + kSgKeys * kSgRow;               // [32 slots][kSgRow]
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
  const int tid = threadIdx.x, lane = tid & 63, r = lane & 15, c = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h0 = w * HW;
  const bool wave_on = h0 < H;
  const int qpos = pos0 + r;
  const int tswz = (r >> 2) & 3;

  sg_bf16x8 qf[HW][ND];
  float k3[HW];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int h = h0 + hh;
    k3[hh] = h < H ? -((CAP ? a.cap : 0.f) + a.bias[h]) * kLog2e : 0.f;
#pragma unroll
    for (int st = 0; st < ND; ++st) {
      qf[hh][st] = zero_frag();
      if (r < ntok && h < H && st * 32 + 8 * c < dim)
        qf[hh][st] = ld_frag(q + (static_cast<int64_t>(row0 + qo + r) * H + h) * dim + st * 32 + 8 * c);
    }
  }
  const float k1 = CAP ? 2.0f * kLog2e * a.scale / a.cap : -kLog2e * a.scale;
  const float k2 = 2.0f * a.cap * kLog2e;
  // B operand of the mix: column = output slot, rows = input slots 8 c .. 8 c + 7
  sg_bf16x8 tf[2];
#pragma unroll
  for (int ht = 0; ht < 2; ++ht) {
    const int so = ht * 16 + r;
    const int ho = (so >> 2) * HW + (so & 3);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int si = 8 * c + j;
      const int hi = (si >> 2) * HW + (si & 3);
      const bool ok = (so & 3) < HW && ho < H && (si & 3) < HW && hi < H;
      tf[ht][j] = static_cast<__bf16>(ok ? a.talk[ho * H + hi] : 0.f);
    }
  }
  const int nht = (H - 1) / HW >= 4 ? 2 : 1;   // output slot tiles in use
  sg_f32x4 O[HW][NV];
#pragma unroll
  for (int hh = 0; hh < HW; ++hh)
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) O[hh][vt] = sg_f32x4{0.f, 0.f, 0.f, 0.f};

  const int* bt = a.block_tables + static_cast<int64_t>(s) * a.bt_width;
  const int64_t kpage = static_cast<int64_t>(G) * bs * dim, vpage = static_cast<int64_t>(G) * vdim * bs;
  const int shift = a.bs_shift, bmask = bs - 1;
  auto page_at = [&](int key) -> int64_t { return key < kend ? bt[key >> shift] : 0; };

  auto scores = [&](int k0, int64_t pg0, int64_t pg1) {
    if (!wave_on) {
      if (k0 == 0) {   // this wave's slots never hold a head: zero them once
        const sg_bf16x4 z = {static_cast<__bf16>(0.f), static_cast<__bf16>(0.f),
                             static_cast<__bf16>(0.f), static_cast<__bf16>(0.f)};
        for (int i = 0; i < 8; ++i) {
          const int key = (i >> 2) * 16 + 4 * c + (i & 3);
          const int o = key * kSgRow + r * 32 + (((w >> 1) ^ tswz) << 3) + (w & 1) * 4;
          *reinterpret_cast<sg_bf16x4*>(w_hi + o) = z;
          *reinterpret_cast<sg_bf16x4*>(w_lo + o) = z;
        }
      }
      return;
    }
    const bool edge = k0 + kSgKeys - 1 > pos0;   // some key lies after the first query token
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      const int key = k0 + sub * 16 + r;
      const __bf16* kb = k_cache + (sub ? pg1 : pg0) * kpage + static_cast<int64_t>(key & bmask) * dim + 8 * c;
      sg_bf16x8 kf[ND];
      float wt[4][4];
#pragma unroll
      for (int hh = 0; hh < 4; ++hh) {
        if (hh >= HW) {
#pragma unroll
          for (int i = 0; i < 4; ++i) wt[hh][i] = 0.f;
          continue;
        }
        const int h = h0 + hh;
        const int g = h / rep;
        if (h < H && (hh == 0 || g != (h - 1) / rep)) {   // wave-uniform: a new KV head
#pragma unroll
          for (int st = 0; st < ND; ++st) {
            kf[st] = zero_frag();
            if (key < kend && st * 32 + 8 * c < dim)
              kf[st] = ld_frag(kb + static_cast<int64_t>(g) * bs * dim + st * 32);
          }
        }
        sg_f32x4 S = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int st = 0; st < ND; ++st)
          S = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[st], qf[hh < HW ? hh : 0][st], S, 0, 0, 0);
        const float b = k3[hh < HW ? hh : 0];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float x = h < H ? sig_weight<CAP>(S[i], k1, k2, b) : 0.f;
          if (edge && k0 + sub * 16 + 4 * c + i > qpos) x = 0.f;
          wt[hh][i] = x;
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int kk = sub * 16 + 4 * c + i;
        const int o = kk * kSgRow + r * 32 + (((w >> 1) ^ tswz) << 3) + (w & 1) * 4;
        sg_bf16x4 hi, lo;
#pragma unroll
        for (int hh = 0; hh < 4; ++hh) {
          hi[hh] = static_cast<__bf16>(wt[hh][i]);
          lo[hh] = static_cast<__bf16>(wt[hh][i] - static_cast<float>(hi[hh]));
        }
        *reinterpret_cast<sg_bf16x4*>(w_hi + o) = hi;
        *reinterpret_cast<sg_bf16x4*>(w_lo + o) = lo;
      }
    }
  };

  int64_t pk0 = page_at(r), pk1 = page_at(16 + r), pv = page_at(8 * c);
  scores(0, pk0, pk1);
  for (int k0 = 0; k0 < kend; k0 += kSgKeys) {
    __syncthreads();
    const int nk = k0 + kSgKeys;
    pk0 = page_at(nk + r);
    pk1 = page_at(nk + 16 + r);
    // B: the wave mixes the pairs of tokens 2 w and 2 w + 1
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      const int t = 2 * w + tt, swz = (t >> 2) & 3;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int o = (half * 16 + r) * kSgRow + t * 32 + ((c ^ swz) << 3);
        const sg_bf16x8 ah = ld_frag(w_hi + o), al = ld_frag(w_lo + o);
#pragma unroll
        for (int ht = 0; ht < 2; ++ht) {
          if (ht < nht) {
            sg_f32x4 D = {0.f, 0.f, 0.f, 0.f};
            D = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, tf[ht], D, 0, 0, 0);
            D = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, tf[ht], D, 0, 0, 0);
            sg_bf16x4 e;
#pragma unroll
            for (int i = 0; i < 4; ++i) e[i] = static_cast<__bf16>(D[i]);
            *reinterpret_cast<sg_bf16x4*>(mixed + (ht * 16 + r) * kSgRow + t * 32 +
                                          (((half * 2 + (c >> 1)) ^ swz) << 3) + (c & 1) * 4) = e;
          }
        }
      }
    }
    __syncthreads();
    if (wave_on) {   // C
      const int t8 = k0 + 8 * c;
      sg_bf16x8 pf[HW];
#pragma unroll
      for (int hh = 0; hh < HW; ++hh)
        pf[hh] = ld_frag(mixed + (4 * w + hh) * kSgRow + r * 32 + ((c ^ tswz) << 3));
      const __bf16* vb = v_cache + pv * vpage + (t8 & bmask) + static_cast<int64_t>(r) * bs;
#pragma unroll
      for (int vt = 0; vt < NV; ++vt) {
        if (vt < nv) {
          sg_bf16x8 vf = zero_frag();
#pragma unroll
          for (int hh = 0; hh < HW; ++hh) {
            const int h = h0 + hh;
            if (h < H) {
              const int g = h / rep;
              if (hh == 0 || g != (h - 1) / rep)
                vf = ld_v(vb + (static_cast<int64_t>(g) * vdim + vt * 16) * bs, t8, kend);
              O[hh][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[hh], O[hh][vt], 0, 0, 0);
            }
          }
        }
      }
    }
    pv = page_at(nk + 8 * c);
    if (nk < kend) scores(nk, pk0, pk1);
  }
  if (!wave_on || r >= ntok) return;
#pragma unroll
  for (int hh = 0; hh < HW; ++hh) {
    const int h = h0 + hh;
    if (h < H) {
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

// One workgroup of four waves per (decode sequence, 64-key partition), all heads.
template <int ND, bool CAP>   // dim <= 32 ND
__global__ void __launch_bounds__(256)
sigmoid_attention_decode_kernel(const __bf16* __restrict__ q, const __bf16* __restrict__ k_cache,
                                const __bf16* __restrict__ v_cache, SigArgs a) {
  extern __shared__ __attribute__((aligned(16))) char sg_smem[];
  const int H = a.H, G = a.G, dim = a.dim, vdim = a.vdim, bs = a.block_size, HS = H + 1;
  constexpr int PR = kSgPart + 8;
  __bf16* mixed = reinterpret_cast<__bf16*>(sg_smem);                       // [H][72]
  float* wts = reinterpret_cast<float*>(sg_smem + sizeof(__bf16) * H * PR); // [64 keys][H + 1]
  const int s = blockIdx.x, kbeg = blockIdx.y * kSgPart;
  const int kvlen = a.seq_kvlen[s];
  const int kend = min(kvlen, kbeg + kSgPart);
  if (kbeg >= kend) return;
  const int rep = H / G, ct = (rep + 15) >> 4;
  const int lane = threadIdx.x & 63, r = lane & 15, c = lane >> 4;
  const int w = __builtin_amdgcn_readfirstlane(static_cast<int>(threadIdx.x) >> 6);
  const int* bt = a.block_tables + static_cast<int64_t>(s) * a.bt_width;
  const int64_t row = a.seq_qstart[s];
  const float k1 = CAP ? 2.0f * kLog2e * a.scale / a.cap : -kLog2e * a.scale;
  const float k2 = 2.0f * a.cap * kLog2e;
  const int shift = a.bs_shift, bmask = bs - 1;
  // wave w scores keys 16 w .. 16 w + 15 of the partition for every KV head
  {
    const int key = kbeg + 16 * w + r;
    const bool live = key < kend;
    const __bf16* kb = k_cache + (live ? static_cast<int64_t>(bt[key >> shift]) : 0) * G * bs * dim +
                       static_cast<int64_t>(key & bmask) * dim + 8 * c;
    for (int j = 0; j < G * ct; ++j) {
      const int g = j / ct, hl = (j - g * ct) * 16 + r, h = g * rep + hl;
      const bool hok = hl < rep;
      sg_f32x4 S = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < ND; ++st) {
        sg_bf16x8 kf = zero_frag(), qf = zero_frag();
        if (st * 32 + 8 * c < dim) {
          if (live) kf = ld_frag(kb + static_cast<int64_t>(g) * bs * dim + st * 32);
          if (hok) qf = ld_frag(q + (row * H + h) * dim + st * 32 + 8 * c);
        }
        S = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, S, 0, 0, 0);
      }
      if (hok) {
        const float k3 = -((CAP ? a.cap : 0.f) + a.bias[h]) * kLog2e;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int kk = 16 * w + 4 * c + i;
          wts[kk * HS + h] = kbeg + kk < kend ? sig_weight<CAP>(S[i], k1, k2, k3) : 0.f;
        }
      }
    }
  }
  __syncthreads();
  // lane = key, four output heads per pass of a wave
  for (int hb = 4 * w; hb < H; hb += 16) {
    float m[4] = {0.f, 0.f, 0.f, 0.f};
    const float* tr[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) tr[e] = a.talk + static_cast<int64_t>(min(hb + e, H - 1)) * H;
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
  for (int j = w; j < G * ct * nv; j += 4) {
    const int vt = j % nv, gc = j / nv;
    const int g = gc / ct, hl = (gc - g * ct) * 16 + r, h = g * rep + hl;
    sg_f32x4 O = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const int t8 = kbeg + ks * 32 + 8 * c;
      sg_bf16x8 vf = zero_frag();
      if (t8 < kend)
        vf = ld_v(v_cache + (static_cast<int64_t>(bt[t8 >> shift]) * G + g) * vdim * bs +
                      static_cast<int64_t>(vt * 16 + r) * bs + (t8 & bmask),
                  t8, kend);
      const sg_bf16x8 pf = hl < rep ? ld_frag(mixed + h * PR + ks * 32 + 8 * c) : zero_frag();
      O = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf, O, 0, 0, 0);
    }
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

template <int HW, int ND, int NV, bool CAP>
int sg_launch_prefill(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
                      int num_tiles, hipStream_t st) {
  const size_t smem = sizeof(__bf16) * (2 * kSgKeys + kSgSlots) * kSgRow;
  static bool opted = false;
  if (!opted) {
    if (int rc = sg_smem_opt_in(sigmoid_attention_mfma_kernel<HW, ND, NV, CAP>, smem)) return rc;
    opted = true;
  }
  hipLaunchKernelGGL((sigmoid_attention_mfma_kernel<HW, ND, NV, CAP>),
                     dim3(num_tiles * (kSgTile / kSgTok)), dim3(512), smem, st,
                     static_cast<__bf16*>(out), static_cast<const __bf16*>(q),
                     static_cast<const __bf16*>(k), static_cast<const __bf16*>(v), a);
  return static_cast<int>(hipGetLastError());
}

template <int HW, bool CAP>
int sg_prefill_dims(void* out, const void* q, const void* k, const void* v, const SigArgs& a,
                    int num_tiles, hipStream_t st) {
  if (a.dim <= 64 && a.vdim <= 64) return sg_launch_prefill<HW, 2, 4, CAP>(out, q, k, v, a, num_tiles, st);
  return sg_launch_prefill<HW, 4, 8, CAP>(out, q, k, v, a, num_tiles, st);
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
  // H <= 64: at most 9 KB of mixed weights and 17 KB of weights
  const size_t smem = sizeof(__bf16) * a.H * (kSgPart + 8) + sizeof(float) * kSgPart * (a.H + 1);
  hipLaunchKernelGGL((sigmoid_attention_decode_kernel<ND, CAP>), dim3(num_decode, parts), dim3(256),
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
                                      const float* talk, int use_mfma, int dtype, hipStream_t st) {
  if (num_tiles <= 0 && num_decode <= 0) return 0;
  if (G <= 0 || H % G != 0 || cap < 0.f) return -1;
  const int parts = (max_decode_kv + kSgPart - 1) / kSgPart;
  if (num_decode > 0 && (parts < 1 || parts > max_parts || part == nullptr)) return -1;
  int bs_shift = 0;
  while ((1 << bs_shift) < block_size) ++bs_shift;
  const SigArgs a{block_tables, seq_kvlen, seq_qstart, tile_seq, tile_qoff, part, bias, talk,
                  bt_width, H, G, dim, vdim, block_size, bs_shift, max_parts, 0, scale, cap};
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
