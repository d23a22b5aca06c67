// Prefill of grouped-query attention with a sliding window and attention sinks on MFMA
// (layouts and semantics in gqa.hip; 128-row query tiles from the runner's tile list).
//
// Workgroup: 4 waves = HB query heads of one key/value head x RW = 4 / HB groups of 32
// query rows, so every 64-key K / V tile staged in LDS feeds 4 waves whatever the group
// size.  A wave is 32 rows of one head:
//   S^T = K Q^T      lane (row l & 31, hi = l >> 5) holds 32 of its row's 64 scores
//   O^T += V^T P^T   the lane's own scores are the B operand; V^T fragments by
//                    ds_read_b64_tr_b16 from the row-major tile, the keys of a k-step
//                    permuted the same way on both sides
// Tiles go global -> LDS by LDS-DMA, two stages, one barrier a tile; the tiles of kept first
// keys come before those of the block's window, the ones between are not visited, and tiles
// of which a wave sees nothing are not computed.  The
// sink is the initial term of the online softmax (maximum = sink, sum = 1).  Caps and
// distance biases (score.h) are applied to the score tile in registers; the head's gate joins
// the last division.  Capped scores that only lose by their distance are bounded: exp(s) fits
// fp32 as it is, and neither a running maximum nor a rescaling is needed.  A tile is then
// worked on in halves of 32 keys, its biases are a table of distances in LDS, and the
// denominator sums the same rounded P as the output.
#include <type_traits>

#include "mask.h"
#include "score.h"

using namespace omnia;

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ float16v mfma32(short8 a, short8 b, float16v c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

// chunk XOR of row `row` in a [64][W] bf16 image: 16 consecutive rows, read at one
// column, fall on 16 different 16-B slots of the banks.  What the row stride does not
// spread by itself (W 128-multiples: nothing, 64: two rows, 32: four), the XOR does.
template <int W>
__device__ __forceinline__ int swz(int row) {
  constexpr int top = W % 128 == 0 ? 3 : W % 64 == 0 ? 2 : 0;
  const int a = top == 3 ? row & 3 : top == 2 ? (row >> 1) & 1 : 0;
  return (a << 2) | ((row >> 2) & 3);
}
// byte offset of 16-B chunk ch of a row
template <int W>
__device__ __forceinline__ int img(int row, int ch) {
  return row * (2 * W) + 16 * (ch ^ swz<W>(row));
}

struct Args {
  bf16_t* out;        // [T, H, DV]
  const bf16_t* q;    // [T, H, DK]
  const bf16_t* kc;
  const bf16_t* vc;
  const int* block_tables;
  const int* q_start;
  const int* seq_lens;
  const int* tile_seq;
  const int* tile_q0;
  const float* sinks;  // [H] or null
  const float* gate;   // [T, H] or null
  int bt_stride, n_tiles, H, G, hb_lg, page_lg;
  Mask mask;
  Score2 score;
};

// KEEP: windows hold the sequence's first p.mask.keep keys as well.  SHAPE: scores are plain
// (0), capped or biased (1), capped and biased within bounds (2)
template <int DK, int DV, bool KEEP, int SHAPE>
__global__ __launch_bounds__(256, DK + DV <= 256 ? 2 : 1) void prefill_kernel(Args p) {
  // two K | V stages as separate objects: reads of one cannot alias the DMA into the other
  __shared__ __attribute__((aligned(16))) char st0[128 * (DK + DV)];
  __shared__ __attribute__((aligned(16))) char st1[128 * (DK + DV)];
  constexpr int kMaxPages = 1024;  // pages of the visible range staged in LDS
  __shared__ int pg_lds[kMaxPages];
  // SHAPE 2: per wave, cap - bias of the 95 distances between its rows and a tile's keys
  __shared__ float dist_lds[SHAPE == 2 ? 4 : 1][96];

  const int HB = 1 << p.hb_lg, group = p.H / p.G;
  // blocks of one key/value head are neighbours: (head block, tile, sub-tile)
  const int id = xcd_remap(blockIdx.x, gridDim.x);
  const int sub = id & (HB - 1), rest = id >> p.hb_lg;
  const int hblk = rest / p.n_tiles, tile = rest - hblk * p.n_tiles;
  const int s = p.tile_seq[tile];
  const int qs = p.q_start[s], qlen = p.q_start[s + 1] - qs;
  const int rows = 128 >> p.hb_lg;  // of this block: the tile has HB sub-tiles
  const int b0 = p.tile_q0[tile] + sub * rows;
  if (b0 >= qlen) return;
  const int off = p.seq_lens[s] - qlen;  // position of the portion's first row
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, ql = lane & 31, hi = lane >> 5;
  const int h = hblk * HB + (w & (HB - 1)), kvh = hblk * HB / group;
  const int* bt = p.block_tables + (int64_t)s * p.bt_stride;
  const int BS = 1 << p.page_lg, pmask = BS - 1;

  const int q0 = b0 + 32 * (w >> p.hb_lg);  // this wave's first row
  const int qr = q0 + ql;
  const bool row_ok = qr < qlen;
  const int qr_c = min(qr, qlen - 1), qpos = off + qr_c;
  const int wmin = off + min(q0, qlen - 1), wmax = off + min(q0 + 31, qlen - 1);
  short8 qf[DK / 16];
  {
    const bf16_t* qrow = p.q + ((int64_t)(qs + qr_c) * p.H + h) * DK + 8 * hi;
#pragma unroll
    for (int ks = 0; ks < DK / 16; ++ks) qf[ks] = *reinterpret_cast<const short8*>(qrow + 16 * ks);
  }
  const int keep = KEEP ? p.mask.keep : 0, qlo = p.mask.lo(qpos);
  const int lo_min = p.mask.lo(wmin), lo_max = p.mask.lo(wmax);
  const int kv_end = off + min(b0 + rows, qlen);
  // visited tiles: [0, tk) with kept keys, then the window's [t0, t1)
  const int t0 = p.mask.lo(off + b0) >> 6, t1 = (kv_end + 63) >> 6;
  const int tk = KEEP ? min((keep + 63) >> 6, t0) : 0, nt = tk + t1 - t0;
  auto tile_of = [&](int j) { return KEEP && j < tk ? j : t0 + j - tk; };
  // staged pages: those of the kept tiles, then the window's from pg0 on
  const int nkp = ((tk << 6) + BS - 1) >> p.page_lg;
  const int pg0 = (t0 << 6) >> p.page_lg;
  const int npg = min(nkp + ((kv_end - 1) >> p.page_lg) - pg0 + 1, kMaxPages);
  for (int i = tid; i < npg; i += 256) pg_lds[i] = bt[i < nkp ? i : pg0 + i - nkp];
  __syncthreads();

  typedef __attribute__((address_space(3))) void* lds_ptr_t;
  // one tensor's tile: instruction i of wave w fills 64 consecutive 16-B slots; the image's
  // XOR is applied to the source chunk.  Keys past the end re-read the last one (masked).
  auto dma1 = [&](int t, auto WC, const bf16_t* src, char* dst) {
    constexpr int W = decltype(WC)::value, CPR = W / 8, N = W / 32;
    int64_t at[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int c = (w * N + i) * 64 + lane, row = c / CPR;
      const int key = min(t * 64 + row, kv_end - 1);
      const int pi = (key >> p.page_lg) - (KEEP && t < tk ? 0 : pg0 - nkp);
      const int pl = pg_lds[pi < kMaxPages ? pi : 0];
      const int page = pi < kMaxPages ? pl : bt[key >> p.page_lg];
      at[i] = ((((int64_t)page * p.G + kvh) << p.page_lg) + (key & pmask)) * W +
              8 * ((c - row * CPR) ^ swz<W>(row));
    }
#pragma unroll
    for (int i = 0; i < N; ++i)
      __builtin_amdgcn_global_load_lds((const void*)(src + at[i]),
                                       (lds_ptr_t)(dst + (w * N + i) * 1024), 16, 0, 0);
  };
  auto dma = [&](int t, auto BUF) {
    char* st = decltype(BUF)::value ? st1 : st0;
    dma1(t, std::integral_constant<int, DK>{}, p.kc, st);
    dma1(t, std::integral_constant<int, DV>{}, p.vc, st + 128 * DK);
  };

  const float r1 = SHAPE && p.score.r1 ? p.score.r1[h] : 0.f;
  const float r2 = SHAPE && p.score.r1 ? p.score.r2[h] : 0.f;
  const float to2 = SHAPE ? 1.f : p.score.mul;  // the tile's scores to base 2
  const float sink = p.sinks ? p.sinks[h] * 1.4426950408889634f : -1e30f;
  float m_run = sink;
  float l_run = p.sinks && SHAPE != 2 ? 1.f : 0.f;
  float16v o[DV / 32];
#pragma unroll
  for (int d = 0; d < DV / 32; ++d)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[d][r] = 0.f;
  // transposed-read roles: 16-lane group g covers columns 16 (g & 1) .. +15 of a 32-column
  // block for the k-slot half g >> 1; lane 4 qg + pp addresses key row qg, columns 4 pp ..
  const int g = lane >> 4, qg = (lane & 15) >> 2, pp = lane & 3;

  using B0 = std::integral_constant<int, 0>;
  using B1 = std::integral_constant<int, 1>;
  dma(tile_of(0), B0{});
  __syncthreads();
  auto body = [&](int j, auto BUF) {
    constexpr int buf = decltype(BUF)::value;
    const int t = tile_of(j);
    if (j + 1 < nt) dma(tile_of(j + 1), std::integral_constant<int, 1 - buf>{});
    const char* Kl = buf ? st1 : st0;
    const char* Vl = Kl + 128 * DK;
    const int k0 = t * 64;
    // S^T of 32 keys
    auto scores = [&](int half) {
      float16v a;
#pragma unroll
      for (int r = 0; r < 16; ++r) a[r] = 0.f;
#pragma unroll
      for (int ks = 0; ks < DK / 16; ++ks)
        a = mfma32(*reinterpret_cast<const short8*>(Kl + img<DK>(half * 32 + ql, 2 * ks + hi)),
                   qf[ks], a);
      return a;
    };
    // O^T += V^T P^T over the 16 keys of a k-step
    auto add = [&](int st, short8 pb) {
      typedef short v4s __attribute__((ext_vector_type(4)));
      typedef __attribute__((address_space(3))) v4s* lds_v4s;
      const int kb = (st >> 1) * 32 + 16 * (st & 1) + 4 * (g >> 1) + qg;
#pragma unroll
      for (int d = 0; d < DV / 32; ++d) {
        const int ch = d * 4 + 2 * (g & 1) + (pp >> 1);
        const v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (lds_v4s)(Vl + img<DV>(kb, ch) + 8 * (pp & 1)));
        const v4s hv = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (lds_v4s)(Vl + img<DV>(kb + 8, ch) + 8 * (pp & 1)));
        o[d] = mfma32(__builtin_shufflevector(lo, hv, 0, 1, 2, 3, 4, 5, 6, 7), pb, o[d]);
      }
    };
    // wave-uniform: some row sees some key
    const bool seen = k0 <= wmax && (k0 + 63 >= lo_min || (KEEP && k0 < keep));
    if (SHAPE == 2 && seen) {
      // entry t: distance (first row + 31) - (first key) - t; keys ahead of a row are masked
      float* dist = dist_lds[w];
      const int far = off + q0 + 31 - k0;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int t = lane + 64 * i;
        if (t < 95)
          dist[t] = p.score.cap - r1 * log2_(__builtin_fmaf(r2, (float)max(far - t, 0), 1.f));
      }
      __builtin_amdgcn_wave_barrier();
      const float* mine = dist + 31 - ql + 4 * hi;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        if (k0 + 32 * half > wmax) break;
        float16v sa = scores(half);
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float e = __builtin_amdgcn_exp2f(sa[r] * p.score.mul) + 1.f;
          sa[r] = __builtin_fmaf(-2.f * p.score.cap, __builtin_amdgcn_rcpf(e),
                                 mine[half * 32 + (r & 3) + 8 * (r >> 2)]);
        }
        if (k0 + 63 > wmin || k0 < lo_max) {  // an edge crosses the tile
          const int top = qpos - k0 - 4 * hi, bot = qlo - k0 - 4 * hi;
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int kk = half * 32 + (r & 3) + 8 * (r >> 2);
            sa[r] = kk > top || kk < bot ? -INFINITY : sa[r];
          }
        }
#pragma unroll
        for (int st = 0; st < 2; ++st) {
          short8 pb;
#pragma unroll
          for (int j = 0; j < 8; ++j)
            pb[j] = __builtin_bit_cast(short, (__bf16)__builtin_amdgcn_exp2f(sa[8 * st + j]));
          const uint4v pairs = __builtin_bit_cast(uint4v, pb);
#pragma unroll
          for (int j = 0; j < 4; ++j)
            l_run += __uint_as_float(pairs[j] << 16) + __uint_as_float(pairs[j] & 0xffff0000u);
          add(2 * half + st, pb);
        }
      }
    } else if (seen) {
      float16v sa[2];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
#pragma unroll
        for (int r = 0; r < 16; ++r) sa[half][r] = 0.f;
#pragma unroll
        for (int ks = 0; ks < DK / 16; ++ks)
          sa[half] = mfma32(*reinterpret_cast<const short8*>(Kl + img<DK>(half * 32 + ql, 2 * ks + hi)),
                            qf[ks], sa[half]);
      }
      if constexpr (SHAPE == 1) {
        const float one = __builtin_fmaf(r2, (float)(qpos - k0 - 4 * hi), 1.f);
#pragma unroll
        for (int half = 0; half < 2; ++half)
#pragma unroll
          for (int r = 0; r < 16; ++r) sa[half][r] *= p.score.mul;
        if (p.score.cap > 0.f) {
#pragma unroll
          for (int half = 0; half < 2; ++half)
#pragma unroll
            for (int r = 0; r < 16; ++r) sa[half][r] = p.score.squash(sa[half][r]);
        }
        if (p.score.r1) {  // keys ahead of the row: not a number, masked below
#pragma unroll
          for (int half = 0; half < 2; ++half)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
              const float kk = half * 32 + (r & 3) + 8 * (r >> 2);
              sa[half][r] = __builtin_fmaf(-r1, log2_(__builtin_fmaf(-kk, r2, one)), sa[half][r]);
            }
        }
      }
      float mloc = -INFINITY;
      if (k0 + 63 > wmin || (k0 < lo_max && (!KEEP || k0 + 63 >= keep))) {  // an edge crosses the tile
        const int top = qpos - k0 - 4 * hi, bot = qlo - k0 - 4 * hi, kp = keep - k0 - 4 * hi;
#pragma unroll
        for (int half = 0; half < 2; ++half)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int kk = half * 32 + (r & 3) + 8 * (r >> 2);
            const float v = (kk > top || (kk < bot && (!KEEP || kk >= kp))) ? -INFINITY : sa[half][r];
            sa[half][r] = v;
            mloc = fmaxf(mloc, v);
          }
      } else {
#pragma unroll
        for (int half = 0; half < 2; ++half)
#pragma unroll
          for (int r = 0; r < 16; ++r) mloc = fmaxf(mloc, sa[half][r]);
      }
      mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64)) * to2;
      // the running maximum moves only when a row's grows by more than 2^8
      const bool grow = mloc > m_run + 8.f;
      if (__builtin_amdgcn_ballot_w64(grow)) {
        const float m_new = grow ? mloc : m_run;
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
        l_run *= alpha;
#pragma unroll
        for (int d = 0; d < DV / 32; ++d) o[d] *= alpha;
        m_run = m_new;
      }
      float lsum = 0.f;
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float e = __builtin_amdgcn_exp2f(
              SHAPE ? sa[half][r] - m_run : __builtin_fmaf(sa[half][r], to2, -m_run));
          sa[half][r] = e;
          lsum += e;
        }
      l_run += lsum + __shfl_xor(lsum, 32, 64);
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        short8 pb;
#pragma unroll
        for (int j = 0; j < 8; ++j)
          pb[j] = __builtin_bit_cast(short, (__bf16)sa[st >> 1][8 * (st & 1) + j]);
        add(st, pb);
      }
    }
    __syncthreads();  // the next tile landed and this one is read by all waves
  };
  for (int j = 0; j < nt; j += 2) {
    body(j, B0{});
    if (j + 1 < nt) body(j + 1, B1{});
  }
  if constexpr (SHAPE == 2)
    l_run += __shfl_xor(l_run, 32, 64) + (p.sinks ? __builtin_amdgcn_exp2f(sink) : 0.f);
  if (row_ok) {
    const float inv = (p.gate ? p.gate[(int64_t)(qs + qr) * p.H + h] : 1.f) / l_run;
    bf16_t* orow = p.out + ((int64_t)(qs + qr) * p.H + h) * DV;
#pragma unroll
    for (int d = 0; d < DV / 32; ++d)
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        uint2v pk;
        pk[0] = pack_bf2(o[d][4 * m] * inv, o[d][4 * m + 1] * inv);
        pk[1] = pack_bf2(o[d][4 * m + 2] * inv, o[d][4 * m + 3] * inv);
        *reinterpret_cast<uint2v*>(orow + d * 32 + 8 * m + 4 * hi) = pk;
      }
  }
}

}  // namespace

extern "C" {

// bounded: r1, r2 >= 0 in all heads, the cap at most 40 and sinks of ordinary size
int omnia_gqa_prefill(void* out, const void* q, const void* kc, const void* vc,
                      const int* block_tables, int bt_stride, const int* q_start,
                      const int* seq_lens, const int* tile_seq, const int* tile_q0, int n_tiles,
                      int page, int H, int G, int Dp, int Vp, Mask mask, Score score,
                      const float* sinks, const float* gate, int bounded, hipStream_t s) {
  if (G < 1 || H % G || !mask.ok() || !score.ok()) return -1;
  if (bounded && (!(score.cap > 0.f && score.cap <= 40.f) || !score.r1)) return -5;
  int page_lg = 0;
  while (page_lg < 30 && (1 << page_lg) < page) ++page_lg;
  if ((1 << page_lg) != page) return -2;
  if (n_tiles == 0) return 0;
  const int group = H / G, hb_lg = group % 4 == 0 ? 2 : group % 2 == 0 ? 1 : 0;
  if ((int64_t)n_tiles * H > 2147483647LL) return -4;
  Args a{(bf16_t*)out, (const bf16_t*)q, (const bf16_t*)kc, (const bf16_t*)vc, block_tables,
         q_start, seq_lens, tile_seq, tile_q0, sinks, gate, bt_stride, n_tiles, H, G, hb_lg,
         page_lg, mask, Score2(score)};
  const bool keep = mask.window > 0 && mask.chunk == 0 && mask.keep > 0;
#define OMNIA_GQ(K, V)                                                  \
  if (Dp == K && Vp == V) {                                             \
    if (!score.plain() && keep)                                         \
      prefill_kernel<K, V, true, 1><<<n_tiles * H, 256, 0, s>>>(a);     \
    else if (bounded)                                                   \
      prefill_kernel<K, V, false, 2><<<n_tiles * H, 256, 0, s>>>(a);    \
    else if (!score.plain())                                            \
      prefill_kernel<K, V, false, 1><<<n_tiles * H, 256, 0, s>>>(a);    \
    else if (keep)                                                      \
      prefill_kernel<K, V, true, 0><<<n_tiles * H, 256, 0, s>>>(a);     \
    else                                                                \
      prefill_kernel<K, V, false, 0><<<n_tiles * H, 256, 0, s>>>(a);    \
    return (int)hipGetLastError();                                      \
  }
#define OMNIA_GQV(K) \
  OMNIA_GQ(K, 32) OMNIA_GQ(K, 64) OMNIA_GQ(K, 96) OMNIA_GQ(K, 128) OMNIA_GQ(K, 192) OMNIA_GQ(K, 256)
  OMNIA_GQV(32) OMNIA_GQV(64) OMNIA_GQV(96) OMNIA_GQV(128) OMNIA_GQV(192) OMNIA_GQV(256)
#undef OMNIA_GQV
#undef OMNIA_GQ
  return -3;
}

}  // extern "C"
