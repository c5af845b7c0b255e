// Attention of many query rows over the K/V rows of a prompt, one kernel per
// call: scores, masked softmax and the product with V without the [H, S, L]
// score and probability tensors ever reaching memory.
//
// One pass over the keys with a running maximum (online softmax): per tile of
// 64 keys the scores are formed (rounded to fp16 like the stand-alone product:
// score = fp16(scale * q.k)), the maximum m is raised if needed - the products
// accumulated so far and the sum of exponentials are then multiplied by
// exp(m_old - m_new) -, the weights fp16(exp(score - m)) go into the second
// product as they are, and the division by the sum of exponentials comes last,
// in fp32, before the one rounding of the output.  The separate operators round
// the NORMALISED probability to fp16 instead (p = fp16(exp(score - max) / sum));
// the two differ by at most two half-ulp roundings of a weight, i.e. by
// 2 * 2^-12 * sum_l p[l] |v[l]|, inside the 1e-2 the outputs are held to.  (A first
// version walked the keys twice - maximum and sum first, then the very
// probabilities of the operators - and took twice as long: two exponentials
// per score and the scores computed twice.)
//
// Workgroup = 4 waves = 128 query rows of one head, 32 per wave; the keys come
// through LDS in tiles of 64.  Both products run on v_mfma_f32_32x32x16_f16 in
// the transposed form, so that a lane's accumulator registers belong to ONE
// query:
//   S^T[key, q] = sum_d K[key, d] Q[q, d]      A = K tile (LDS), B = Q (regs)
//   O^T[d, q]   = sum_key V^T[d, key] P^T[key, q]   A = V^T tile (LDS), B = P^T
// Lane l of a wave owns query l % 32.  Of a 32-key block its 16 accumulator
// registers hold the keys 8*(r/4) + 4*(l/32) + r%4, so maximum and sum over
// keys are sums over a lane's own registers (the two lane halves are merged
// after every tile), and the weights it forms are, as they lie, the B
// operand of the second product: registers 8t .. 8t+7 are the eight k values
// of lane half l/32 in k-step t.  The V tile is written to LDS transposed and
// with its keys permuted to that same order (slot 16t + 8h + j holds key
// 16t + 8*(j/4) + 4h + j%4 of the block), so the A operand of the second
// product is one 16-byte LDS read.
//
// The element type is a template parameter: fp16 (Llama-2, the score rounded
// to fp16 as above) or bf16 (scores stay in fp32; weights are rounded once, as
// the operand of the second product).  Query heads may share key/value heads,
// the score factor may grow with the query's position, and a head's output may
// be scaled by the sigmoid of a per-token gate.
//
// A second, small kernel in this file prepares the inputs of the first from
// the projection outputs: RoPE of Q (in place) and K, and the K/V cache write.
#include "../../include/vkl_hip.h"
#include "../../include/vkl_stack.h"
#include "vkl_common.h"

namespace
{
typedef _Float16 half8 __attribute__ ((ext_vector_type (8)));
typedef __bf16 bf8 __attribute__ ((ext_vector_type (8)));
typedef float float16v __attribute__ ((ext_vector_type (16)));
typedef uint32_t u32x2 __attribute__ ((ext_vector_type (2)));

constexpr int kBQ = 128;      // query rows per workgroup
constexpr int kBKey = 64;     // keys per tile
constexpr int kThreads = 256;
constexpr float kNeg = -1.0e30f; // "no key seen yet": finite, so that kNeg - kNeg = 0

struct AttnArgs
{
  const uint16_t *q, *k, *v;
  uint16_t *out;
  int H, S, L, ntq;
  size_t qcs, qhs, kcs, khs, vcs, vhs, ors, ohs;
  float scale;
  int rep;            // query heads per key/value head
  float temp_coef;    // != 0: scale times 1 + coef ln (floor ((pos + 1) / every) + 1)
  int temp_every;
  const float *gate;  // optional [S, gs]: head h's output times sigmoid (gate[s, h])
  size_t gs;
  int chunk, sink;    // CHUNKED kernels: see vkl_attn_prefill_chunked_bf16
};

// the two element types of the operands
struct F16Elem
{
  typedef half8 v8;
  static constexpr bool round_scores = true;
  static __device__ __forceinline__ float16v
  mfma (v8 a, v8 b, float16v c)
  {
    return __builtin_amdgcn_mfma_f32_32x32x16_f16 (a, b, c, 0, 0, 0);
  }
  static __device__ __forceinline__ uint16_t
  bits (float f)
  {
    return vkl::f2h (f);
  }
  typedef _Float16 t;
};

struct Bf16Elem
{
  typedef bf8 v8;
  static constexpr bool round_scores = false;
  static __device__ __forceinline__ float16v
  mfma (v8 a, v8 b, float16v c)
  {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16 (a, b, c, 0, 0, 0);
  }
  static __device__ __forceinline__ uint16_t
  bits (float f)
  {
    return vkl::f2bf (f);
  }
  typedef __bf16 t;
};

__device__ __align__ (16) const uint32_t g_zero16[4] = { 0, 0, 0, 0 };

__device__ __forceinline__ float
fast_exp (float x)
{
  return __builtin_amdgcn_exp2f (x * 1.44269504088896340736f);
}


template <int HD> struct Tile
{
  static constexpr int CPR = HD / 8;                       // 16-byte chunks per row
  static constexpr int KALL = kBKey * CPR, VALL = (kBKey / 2) * CPR;
  static constexpr int KCH = (KALL + kThreads - 1) / kThreads; // K chunks per thread
  static constexpr int VIT = (VALL + kThreads - 1) / kThreads; // (key pair, chunk) items per thread
  // item numbers past the last exist where the tile is not a multiple of the workgroup
  static constexpr bool KRAG = KALL % kThreads != 0, VRAG = VALL % kThreads != 0;
  uint4 k[KCH];
  uint4 v[VIT][2];
};

// K rows [t*64, t*64+64) of the head, as they lie; rows beyond L read zeros
template <int HD>
__device__ __forceinline__ void
load_k (const AttnArgs &a, const uint16_t *kb, int t, Tile<HD> &r)
{
  constexpr int CPR = Tile<HD>::CPR;
  const void *zeros = g_zero16;
#pragma unroll
  for (int i = 0; i < Tile<HD>::KCH; ++i)
    {
      const int c = threadIdx.x + i * kThreads;
      const int row = t * kBKey + c / CPR;
      r.k[i] = vkl::ldg4 (row < a.L && (!Tile<HD>::KRAG || c < Tile<HD>::KALL) ? (const void *)(kb + (size_t)row * a.khs + (c % CPR) * 8)
                                    : zeros);
    }
}

// key of slot s (0..63) of a tile
__device__ __forceinline__ int
slot_key (int s)
{
  const int blk = s >> 5, t = (s >> 4) & 1, h = (s >> 3) & 1, j = s & 7;
  return 32 * blk + 16 * t + 8 * (j >> 2) + 4 * h + (j & 3);
}

template <int HD>
__device__ __forceinline__ void
load_v (const AttnArgs &a, const uint16_t *vb, int t, Tile<HD> &r)
{
  const void *zeros = g_zero16;
#pragma unroll
  for (int i = 0; i < Tile<HD>::VIT; ++i)
    {
      const int it = threadIdx.x + i * kThreads;
      const int pair = it & 31, dc = it >> 5;
      // slots 2*pair and 2*pair+1 hold two adjacent keys
      const int row = t * kBKey + slot_key (2 * pair);
      const bool in = !Tile<HD>::VRAG || it < Tile<HD>::VALL;
      r.v[i][0] = vkl::ldg4 (row < a.L && in ? (const void *)(vb + (size_t)row * a.vhs + dc * 8) : zeros);
      r.v[i][1] = vkl::ldg4 (row + 1 < a.L && in ? (const void *)(vb + (size_t)(row + 1) * a.vhs + dc * 8)
                                           : zeros);
    }
}

template <int HD>
__device__ __forceinline__ void
store_k (const Tile<HD> &r, uint16_t *Ks)
{
  constexpr int CPR = Tile<HD>::CPR, LDK = HD + 8;
#pragma unroll
  for (int i = 0; i < Tile<HD>::KCH; ++i)
    {
      const int c = threadIdx.x + i * kThreads;
      if (Tile<HD>::KRAG && c >= Tile<HD>::KALL)
        continue;
      *(uint4 *)(Ks + (c / CPR) * LDK + (c % CPR) * 8) = r.k[i];
    }
}

// V^T: row = d, column = slot; a thread writes the two keys of its pair as one
// 32-bit word per d
template <int HD>
__device__ __forceinline__ void
store_v (const Tile<HD> &r, uint16_t *Vt)
{
  constexpr int LDV = kBKey + 8;
#pragma unroll
  for (int i = 0; i < Tile<HD>::VIT; ++i)
    {
      const int it = threadIdx.x + i * kThreads;
      const int pair = it & 31, dc = it >> 5;
      if (Tile<HD>::VRAG && it >= Tile<HD>::VALL)
        continue;
      const uint32_t va[4] = { r.v[i][0].x, r.v[i][0].y, r.v[i][0].z, r.v[i][0].w };
      const uint32_t vb[4] = { r.v[i][1].x, r.v[i][1].y, r.v[i][1].z, r.v[i][1].w };
      uint32_t *dst = (uint32_t *)(Vt + (size_t)(dc * 8) * LDV + 2 * pair);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        {
          dst[(2 * e) * (LDV / 2)] = (va[e] & 0xffffu) | (vb[e] << 16);
          dst[(2 * e + 1) * (LDV / 2)] = (va[e] >> 16) | (vb[e] & 0xffff0000u);
        }
    }
}

// S^T of one 32-key block: rows = keys 32*blk .. +31 of the tile in LDS
template <int HD, class E>
__device__ __forceinline__ float16v
score_block (const uint16_t *Ks, int blk, const typename E::v8 (&qf)[HD / 16], int lane)
{
  constexpr int LDK = HD + 8;
  float16v acc;
#pragma unroll
  for (int r = 0; r < 16; ++r)
    acc[r] = 0.f;
  const uint16_t *kp = Ks + (32 * blk + (lane & 31)) * LDK + (lane >> 5) * 8;
#pragma unroll
  for (int kt = 0; kt < HD / 16; ++kt)
    acc = E::mfma (*(const typename E::v8 *)(kp + kt * 16), qf[kt], acc);
  return acc;
}

// (heads wider than 128 values: one workgroup per compute unit, twice the registers)
// CHUNKED: a query sees keys from the start of its own chunk of positions on, and
// the softmax may have a sink (a score of 0 without a value)
template <int HD, class E, bool CHUNKED = false>
__global__ __launch_bounds__ (kThreads, HD <= 128 ? 2 : 1) void
attn_prefill_kernel (const AttnArgs a)
{
  typedef typename E::v8 v8;
  constexpr int KT = HD / 16, DB = HD / 32;
  constexpr int LDK = HD + 8, LDV = kBKey + 8;
  __shared__ __align__ (16) uint16_t Ks[kBKey * LDK];
  __shared__ __align__ (16) uint16_t Vt[HD * LDV];

  // Heavy query tiles (the last ones: most keys) first.  With a head count
  // that is a multiple of 8 the workgroups of one head share id % 8, which
  // keeps the head's K and V in the L2 of one XCD.
  const int b = blockIdx.x;
  int head, qt;
  if ((a.H & 7) == 0)
    {
      // j: position in the XCD's queue.  Its 32 compute units take the first
      // 32 workgroups, then the next 32 beside them, and so on: every other
      // such layer runs the tiles in the opposite order, so that a heavy tile
      // and a light one share a compute unit.
      const int j = b >> 3;
      head = (b & 7) + 8 * (j / a.ntq);
      qt = ((j >> 5) & 1) ? j % a.ntq : a.ntq - 1 - (j % a.ntq);
    }
  else
    {
      head = b / a.ntq;
      qt = a.ntq - 1 - (b % a.ntq);
    }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lq = lane & 31, hh = lane >> 5;
  const int q0 = qt * kBQ;
  const int qrow = q0 + wave * 32 + lq; // this lane's query
  const int shift = a.L - a.S;          // key l is visible iff l <= qrow + shift
  const int kmax = min (a.L, q0 + kBQ + shift);
  const int ntile = (kmax + kBKey - 1) / kBKey;
  const int wave_last = q0 + wave * 32 + 31 + shift; // last key any query of the wave sees
  // first key of the chunk of this lane's query, of the wave's first and last
  auto chunk_start = [&] (int row) { return CHUNKED && a.chunk ? (row + shift) / a.chunk * a.chunk : 0; };
  const int klow = chunk_start (qrow), wave_low = chunk_start (q0 + wave * 32);
  const int wave_high = chunk_start (q0 + wave * 32 + 31);
  const int t0 = CHUNKED ? chunk_start (q0) / kBKey : 0;
  const int kvh = E::round_scores ? head : head / a.rep;
  const uint16_t *kb = a.k + (size_t)kvh * a.kcs;
  const uint16_t *vb = a.v + (size_t)kvh * a.vcs;
  // this query's score factor
  float scale = a.scale;
  if (!E::round_scores && a.temp_coef != 0.f)
    scale *= 1.0f + a.temp_coef * logf ((float)((qrow + shift + 1) / a.temp_every + 1));

  v8 qf[KT];
  {
    const uint16_t *qp = a.q + (size_t)head * a.qcs + (size_t)min (qrow, a.S - 1) * a.qhs + hh * 8;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
      qf[kt] = __builtin_bit_cast (v8, vkl::ldg4 (qp + kt * 16));
  }

  Tile<HD> tl;
  // One pass over the keys with a running maximum: the accumulated products
  // and the sum of exponentials are rescaled whenever the maximum grows, and
  // the division by the sum comes last.
  // (the sink is a key that every query has seen before the first tile; the sums of
  // the two lane halves are added at the end, one of them has it)
  // (a tile may hold no key of a query's chunk: its first maximum lies far above the
  // score of a hidden key, whose weight is then zero)
  float m = !CHUNKED ? kNeg : a.sink ? 0.f : 0.1f * kNeg, sum = CHUNKED && a.sink && hh == 0 ? 1.f : 0.f;
  float16v oacc[DB];
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int r = 0; r < 16; ++r)
      oacc[db][r] = 0.f;
  load_k<HD> (a, kb, t0, tl);
  load_v<HD> (a, vb, t0, tl);
  for (int t = t0; t < ntile; ++t)
    {
      __syncthreads ();
      store_k<HD> (tl, Ks);
      store_v<HD> (tl, Vt);
      __syncthreads ();
      if (t + 1 < ntile)
        {
          load_k<HD> (a, kb, t + 1, tl);
          load_v<HD> (a, vb, t + 1, tl);
        }
      if (t * kBKey > wave_last || (CHUNKED && t * kBKey + kBKey <= wave_low))
        continue;
      // scores of the tile's 64 keys, rounded to fp16 like the stand-alone
      // product; a key the query must not see counts as "never seen"
      float sv[2][16];
      float bm = kNeg;
      const bool inner = t * kBKey + kBKey - 1 <= q0 + wave * 32 + shift // every key visible to every query of the wave
                         && (!CHUNKED || t * kBKey >= wave_high);
#pragma unroll
      for (int blk = 0; blk < 2; ++blk)
        {
          const float16v acc = score_block<HD, E> (Ks, blk, qf, lane);
          const int key0 = t * kBKey + 32 * blk + 4 * hh;
#pragma unroll
          for (int r = 0; r < 16; ++r)
            {
              const int key = key0 + 8 * (r >> 2) + (r & 3);
              const float sc = E::round_scores ? vkl::h2f (vkl::f2h (acc[r] * scale)) : acc[r] * scale;
              sv[blk][r] = inner || (key <= qrow + shift && (!CHUNKED || key >= klow)) ? sc : kNeg;
              bm = fmaxf (bm, sv[blk][r]);
            }
        }
      // the two halves of the lanes hold different keys of the same query and
      // feed one product: they need the same maximum
      bm = fmaxf (bm, __shfl_xor (bm, 32, 64));
      const float mn = fmaxf (m, bm);
      if (__builtin_amdgcn_ballot_w64 (mn != m) != 0)
        {
          const float alpha = fast_exp (m - mn); // 0 before the first key, 1 where the maximum stays
          sum *= alpha;
#pragma unroll
          for (int db = 0; db < DB; ++db)
#pragma unroll
            for (int r = 0; r < 16; ++r)
              oacc[db][r] *= alpha;
          m = mn;
        }
      v8 pf[2][2];
#pragma unroll
      for (int blk = 0; blk < 2; ++blk)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          {
            // exp (kNeg - m) = 0.  The sum takes the weight as the product
            // below consumes it, rounded to fp16: the weights then add up to
            // one exactly.
            const typename E::t e = (typename E::t)fast_exp (sv[blk][r] - m);
            sum += (float)e;
            pf[blk][r >> 3][r & 7] = e;
          }
#pragma unroll
      for (int db = 0; db < DB; ++db)
        {
          const uint16_t *vp = Vt + (size_t)(32 * db + lq) * LDV + 8 * hh;
#pragma unroll
          for (int blk = 0; blk < 2; ++blk)
#pragma unroll
            for (int t2 = 0; t2 < 2; ++t2)
              oacc[db] = E::mfma (*(const v8 *)(vp + 32 * blk + 16 * t2), pf[blk][t2], oacc[db]);
        }
    }
  // the other half of the lanes has summed the other keys of the same query
  sum += __shfl_xor (sum, 32, 64);
  float inv = 1.0f / sum;
  if (!E::round_scores && a.gate)
    inv = inv / (1.0f + expf (-vkl::ldg (a.gate + (size_t)min (qrow, a.S - 1) * a.gs + head)));
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int r = 0; r < 16; ++r)
      oacc[db][r] *= inv;

  if (qrow >= a.S)
    return;
  uint16_t *op = a.out + (size_t)qrow * a.ors + (size_t)head * a.ohs;
#pragma unroll
  for (int db = 0; db < DB; ++db)
#pragma unroll
    for (int g = 0; g < 4; ++g)
      {
        const int d = 32 * db + 8 * g + 4 * hh;
        u32x2 w;
        w.x = (uint32_t)E::bits (oacc[db][4 * g]) | ((uint32_t)E::bits (oacc[db][4 * g + 1]) << 16);
        w.y = (uint32_t)E::bits (oacc[db][4 * g + 2])
              | ((uint32_t)E::bits (oacc[db][4 * g + 3]) << 16);
        *(VKL_GLOBAL u32x2 *)(op + d) = w;
      }
}
// ---------------------------------------------------------------------------
// RoPE of Q and K and the K/V cache write, straight from the [S, H*hd]
// outputs of the projections: one thread per 8 consecutive elements of a
// (row, head).  Q is rotated in place (the attention kernel reads it with a
// row stride of H*hd), the rotated K and V go to cache rows (k_pos0 + s) %
// maxlen of their head.  Arithmetic of one pair as in the RoPE operator:
// (a, b) -> (fp16(a c - b s), fp16(a s + b c)) with fp32 tables.
// ---------------------------------------------------------------------------
struct RopeKvArgs
{
  uint16_t *q;
  const uint16_t *k, *v;
  uint16_t *kcache, *vcache;
  const float *fc, *fs;
  int S, H, hd, maxlen;
  int q_row0, q_rows;       // rows of q that are rotated, and their positions
  uint32_t q_pos0, k_pos0;  // q row q_row0 + i is at q_pos0 + i; k row s at k_pos0 + s
  size_t rs;                // row stride of q, k, v (elements)
};

__device__ __forceinline__ uint4
rotate8 (const uint4 x, const float *fc, const float *fs)
{
  const uint4 c4 = vkl::ldg4 (fc), s4 = vkl::ldg4 (fs);
  const float c[4] = { __uint_as_float (c4.x), __uint_as_float (c4.y), __uint_as_float (c4.z),
                       __uint_as_float (c4.w) };
  const float sn[4] = { __uint_as_float (s4.x), __uint_as_float (s4.y), __uint_as_float (s4.z),
                        __uint_as_float (s4.w) };
  const uint32_t w[4] = { x.x, x.y, x.z, x.w };
  uint32_t o[4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
    {
      const float a = vkl::h2f ((uint16_t)(w[j] & 0xffff)), b = vkl::h2f ((uint16_t)(w[j] >> 16));
      const float r0 = a * c[j] - b * sn[j];
      const float r1 = a * sn[j] + b * c[j];
      o[j] = (uint32_t)vkl::f2h (r0) | ((uint32_t)vkl::f2h (r1) << 16);
    }
  return make_uint4 (o[0], o[1], o[2], o[3]);
}

__global__ __launch_bounds__ (256) void
rope_kvwrite_kernel (const RopeKvArgs a, size_t total)
{
  const size_t t = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (t >= total)
    return;
  const int cpr = a.hd / 8;
  const int c = (int)(t % cpr);
  const int h = (int)((t / cpr) % a.H);
  const int s = (int)(t / ((size_t)cpr * a.H));
  const size_t src = (size_t)s * a.rs + (size_t)h * a.hd + c * 8;
  const int half = a.hd / 2;
  const uint32_t kpos = a.k_pos0 + (uint32_t)s;
  const size_t dst = ((size_t)h * a.maxlen + kpos % (uint32_t)a.maxlen) * a.hd + c * 8;
  const uint4 kr = rotate8 (vkl::ldg4 (a.k + src), a.fc + (size_t)kpos * half + c * 4,
                            a.fs + (size_t)kpos * half + c * 4);
  *(uint4 *)(a.kcache + dst) = kr;
  *(uint4 *)(a.vcache + dst) = vkl::ldg4 (a.v + src);
  if (s >= a.q_row0 && s < a.q_row0 + a.q_rows)
    {
      const uint32_t qpos = a.q_pos0 + (uint32_t)(s - a.q_row0);
      *(uint4 *)(a.q + src) = rotate8 (vkl::ldg4 (a.q + src), a.fc + (size_t)qpos * half + c * 4,
                                       a.fs + (size_t)qpos * half + c * 4);
    }
}
} // namespace

extern "C" int
vkl_rope_kvwrite_f16 (void *q, const void *k, const void *v, int S, int H,
                      int hd, size_t row_stride, int q_row0, int q_rows,
                      uint32_t q_pos0, uint32_t k_pos0, const float *freqc,
                      const float *freqs, int table_rows, void *kcache,
                      void *vcache, int maxlen, void *stream)
{
  VKL_CHECK_ARG (q && k && v && freqc && freqs && kcache && vcache);
  VKL_CHECK_ARG (S > 0 && H > 0 && hd > 0 && (hd % 8) == 0 && maxlen > 0 && S <= maxlen);
  VKL_CHECK_ARG (q_row0 >= 0 && q_rows >= 0 && q_row0 + q_rows <= S);
  // every position must have a row in the cos / sin tables
  VKL_CHECK_ARG ((size_t)k_pos0 + S <= (size_t)table_rows
                 && (size_t)q_pos0 + q_rows <= (size_t)table_rows);
  VKL_CHECK_ARG ((row_stride % 8) == 0 && row_stride >= (size_t)H * hd);
  VKL_CHECK_ARG (((uintptr_t)q % 16) == 0 && ((uintptr_t)k % 16) == 0 && ((uintptr_t)v % 16) == 0
                 && ((uintptr_t)kcache % 16) == 0 && ((uintptr_t)vcache % 16) == 0
                 && ((uintptr_t)freqc % 16) == 0 && ((uintptr_t)freqs % 16) == 0);
  RopeKvArgs a;
  a.q = (uint16_t *)q, a.k = (const uint16_t *)k, a.v = (const uint16_t *)v;
  a.kcache = (uint16_t *)kcache, a.vcache = (uint16_t *)vcache;
  a.fc = freqc, a.fs = freqs;
  a.S = S, a.H = H, a.hd = hd, a.maxlen = maxlen;
  a.q_row0 = q_row0, a.q_rows = q_rows, a.q_pos0 = q_pos0, a.k_pos0 = k_pos0;
  a.rs = row_stride;
  const size_t total = (size_t)S * H * (hd / 8);
  rope_kvwrite_kernel<<<dim3 ((unsigned)((total + 255) / 256)), dim3 (256), 0, (hipStream_t)stream>>> (
      a, total);
  return vkl_launch_status ();
}

extern "C" int
vkl_attn_prefill_causal_f16 (const void *q, const void *k, const void *v,
                             int H, int S, int L, int hd, size_t qcs,
                             size_t qhs, size_t kcs, size_t khs, size_t vcs,
                             size_t vhs, float scale, void *out, size_t ors,
                             size_t ohs, void *stream)
{
  VKL_CHECK_ARG (q && k && v && out);
  VKL_CHECK_ARG (H > 0 && S > 0 && L >= S);
  VKL_CHECK_ARG (hd == 64 || hd == 128);
  // 16-byte vector loads, 8-byte stores
  VKL_CHECK_ARG (((uintptr_t)q % 16) == 0 && ((uintptr_t)k % 16) == 0 && ((uintptr_t)v % 16) == 0
                 && ((uintptr_t)out % 8) == 0);
  VKL_CHECK_ARG ((qcs % 8) == 0 && (qhs % 8) == 0 && (kcs % 8) == 0 && (khs % 8) == 0
                 && (vcs % 8) == 0 && (vhs % 8) == 0 && (ors % 4) == 0 && (ohs % 4) == 0);
  AttnArgs a = {};
  a.rep = 1;
  a.q = (const uint16_t *)q, a.k = (const uint16_t *)k, a.v = (const uint16_t *)v;
  a.out = (uint16_t *)out;
  a.H = H, a.S = S, a.L = L, a.ntq = (S + kBQ - 1) / kBQ;
  a.qcs = qcs, a.qhs = qhs, a.kcs = kcs, a.khs = khs, a.vcs = vcs, a.vhs = vhs;
  a.ors = ors, a.ohs = ohs, a.scale = scale;
  const dim3 grid ((unsigned)(a.ntq * H));
  if (hd == 128)
    attn_prefill_kernel<128, F16Elem><<<grid, dim3 (kThreads), 0, (hipStream_t)stream>>> (a);
  else
    attn_prefill_kernel<64, F16Elem><<<grid, dim3 (kThreads), 0, (hipStream_t)stream>>> (a);
  return vkl_launch_status ();
}

namespace
{
template <bool CHUNKED>
int
launch_prefill_bf16 (const AttnArgs &a, int hd, hipStream_t s)
{
  const dim3 grid ((unsigned)(a.ntq * a.H)), block (kThreads);
  switch (hd)
    {
    case 32: attn_prefill_kernel<32, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 64: attn_prefill_kernel<64, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 96: attn_prefill_kernel<96, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 128: attn_prefill_kernel<128, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 160: attn_prefill_kernel<160, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 192: attn_prefill_kernel<192, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    case 224: attn_prefill_kernel<224, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    default: attn_prefill_kernel<256, Bf16Elem, CHUNKED><<<grid, block, 0, s>>> (a); break;
    }
  return vkl_launch_status ();
}

int
prefill_args_bf16 (AttnArgs &a, const void *q, const void *k, const void *v, int H, int G, int S, int L, int hd,
                   size_t qhs, size_t khs, size_t vhs, float scale, void *out, size_t ors)
{
  VKL_CHECK_ARG (q && k && v && out);
  VKL_CHECK_ARG (H > 0 && G > 0 && (H % G) == 0 && S > 0 && L >= S);
  VKL_CHECK_ARG (hd > 0 && (hd % 32) == 0 && hd <= 256);
  VKL_CHECK_ARG (((uintptr_t)q % 16) == 0 && ((uintptr_t)k % 16) == 0 && ((uintptr_t)v % 16) == 0
                 && ((uintptr_t)out % 8) == 0);
  VKL_CHECK_ARG ((qhs % 8) == 0 && (khs % 8) == 0 && (vhs % 8) == 0 && (ors % 4) == 0);
  VKL_CHECK_ARG (qhs >= (size_t)H * hd && khs >= (size_t)G * hd && vhs >= (size_t)G * hd && ors >= (size_t)H * hd);
  a.q = (const uint16_t *)q, a.k = (const uint16_t *)k, a.v = (const uint16_t *)v;
  a.out = (uint16_t *)out;
  a.H = H, a.S = S, a.L = L, a.ntq = (S + kBQ - 1) / kBQ;
  a.qcs = a.kcs = a.vcs = a.ohs = (size_t)hd;
  a.qhs = qhs, a.khs = khs, a.vhs = vhs, a.ors = ors;
  a.scale = scale, a.rep = H / G;
  return 0;
}
} // namespace

extern "C" int
vkl_attn_prefill_causal_bf16 (const void *q, const void *k, const void *v, int H, int G, int S, int L, int hd,
                              size_t qhs, size_t khs, size_t vhs, float scale, float temp_coef,
                              int temp_every, const float *gate, size_t gs, void *out, size_t ors,
                              void *stream)
{
  AttnArgs a = {};
  if (int e = prefill_args_bf16 (a, q, k, v, H, G, S, L, hd, qhs, khs, vhs, scale, out, ors))
    return e;
  VKL_CHECK_ARG ((temp_coef == 0.f || temp_every > 0) && (!gate || gs >= (size_t)H));
  a.temp_coef = temp_coef, a.temp_every = temp_every, a.gate = gate, a.gs = gs;
  return launch_prefill_bf16<false> (a, hd, (hipStream_t)stream);
}

extern "C" int
vkl_attn_prefill_chunked_bf16 (const void *q, const void *k, const void *v, int H, int G, int S, int L, int hd,
                               size_t qhs, size_t khs, size_t vhs, float scale, int chunk, int sink, void *out,
                               size_t ors, void *stream)
{
  AttnArgs a = {};
  if (int e = prefill_args_bf16 (a, q, k, v, H, G, S, L, hd, qhs, khs, vhs, scale, out, ors))
    return e;
  VKL_CHECK_ARG (chunk >= 0);
  a.chunk = chunk, a.sink = sink;
  return launch_prefill_bf16<true> (a, hd, (hipStream_t)stream);
}
