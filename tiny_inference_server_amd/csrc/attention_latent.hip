// Attention over one shared latent per position on the matrix cores (gfx950, bfloat16): every query head of a row
// attends the same keys (KD channels: the latent and a rotated part) and takes the keys' first VD channels as values.
// Built once per (KD, VD): -DTIS_LATENT=KD*10000+VD.
//
// Pages of 16 slots hold the keys as [slot][KD] and then the values transposed, [VD][slot] (the layout of every
// attention kernel of this engine with one key/value head). 16 columns share their keys, a column being a (row, query head)
// pair. Keys go by in pages:
//   S^T = K . Q^T    keys and queries are the operands of v_mfma_f32_16x16x32_bf16
//   O^T += V^T . P^T the transposed values and the weights, rounded to bfloat16, likewise
// The contraction's order is free as long as both operands agree, so a lane that holds a column's scores of four keys of a
// page feeds exactly those as its share of P^T. Softmax in 32-bit with a running maximum per column. Slots behind a row's
// position are read (their page is mapped) but their scores become -inf and their values zero before any arithmetic.
// A long key range is cut into `n_splits` parts (grid z) whose partial results a second kernel merges. window > 0: a row
// sees its last `window` keys only; pages that no row of an item sees are left out, and slots before the first key any
// row sees (their page may have gone to another request) are treated like those behind the last. sinks (nullable): head h's
// softmax has one more key of score sinks[h], not scaled, without a value.
#include "common.h"

TIS_DEFINE_LAST_ERROR(tis_attention_latent)

#ifndef TIS_LATENT
#define TIS_LATENT 5760512
#endif
static constexpr int KD = TIS_LATENT / 10000, VD = TIS_LATENT % 10000;
static_assert(KD % 8 == 0 && VD % 16 == 0 && VD <= KD && VD >= 16, "key channels in steps of 8, value channels in steps of 16");
static constexpr int DC = (KD + 31) / 32;      // 32-channel chunks of a key
static constexpr int DB = VD / 16;             // 16-channel blocks of a value
static constexpr int PAGE = 16;

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ float quad_max(float v) {      // over the four lanes that share a column
  v = fmaxf(v, __shfl_xor(v, 16, 64));
  return fmaxf(v, __shfl_xor(v, 32, 64));
}
// what a sink of score `sinks[head]` adds to a denominator whose exponentials are 2^(score * log2(e) - m)
__device__ __forceinline__ float sink_share(const float* sinks, int head, float m) {
  return sinks ? exp2f(sinks[head] * 1.4426950408889634f - m) : 0.f;
}
__device__ __forceinline__ float quad_sum(float v) {
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}

// Single rows: a workgroup of four waves takes a row's heads in blocks of 16 and one part of its keys, four pages at a time.
// Wave w multiplies page w's keys with the queries (from LDS, where they lie once for all four); the columns' maxima and the
// weights, rounded to bfloat16, meet in LDS; then every wave adds up all 64 keys for its share of the value channels (every
// fourth block of 16). So a workgroup has everything it needs of four pages on its way at once, in four short chains.
static constexpr int DEC_PAGES = 4, DEC_KEYS = DEC_PAGES * PAGE;
static constexpr int DEC_DB = (DB + 3) / 4;                    // blocks of value channels a wave takes
static constexpr int DQ_STRIDE = KD + 8;                       // elements between two columns' queries in LDS

__global__ __launch_bounds__(256) void latent_decode_kernel(
    const bf16* __restrict__ q, long ldq, const bf16* __restrict__ plane, const int* __restrict__ block_tables, int bt_ld,
    const int* __restrict__ row_seq, const int* __restrict__ positions, bf16* __restrict__ out, long ldo,
    float* __restrict__ part_o, float2* __restrict__ part_ml, int H, float scale_log2, int n_splits, int window,
    const float* __restrict__ sinks) {
  __shared__ __attribute__((aligned(16))) bf16 q_lds[16 * DQ_STRIDE];
  __shared__ bf16x4 p_lds[DEC_PAGES][64];
  __shared__ float col_lds[DEC_PAGES][16];
  const long row = blockIdx.x;
  const int hb = blockIdx.y, split = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), c16 = lane & 15, g = lane >> 4;
  const int pos = positions[row];
  const int* bt = block_tables + (long)row_seq[row] * bt_ld;
  const int head = hb * 16 + c16;
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const int k_lo = window > 0 ? max(0, pos - window + 1) : 0;       // the first key the row sees
  const int c_first = k_lo / DEC_KEYS, n_chunks = pos / DEC_KEYS + 1 - c_first;
  const int per = (n_chunks + n_splits - 1) / n_splits;
  const int c_begin = c_first + split * per, c_end = min(c_first + n_chunks, c_begin + per);
  const long page_stride = (long)PAGE * (KD + VD);
  const int last_page = pos / PAGE, first_page = k_lo / PAGE;

  // (the queries are asked for first and put into LDS once the first keys and values have been asked for, too)
  constexpr int QN = (2 * KD + 255) / 256;
  bf16x8 qreg[QN];
#pragma unroll
  for (int j = 0; j < QN; ++j) {
    const int i = tid + j * 256, col = i / (KD / 8), piece = i % (KD / 8);
    qreg[j] = (i < 2 * KD && hb * 16 + col < H)
                  ? *reinterpret_cast<const bf16x8*>(q + row * ldq + (long)(hb * 16 + col) * KD + piece * 8) : zero8;
  }
  f32x4 o[DEC_DB];
#pragma unroll
  for (int i = 0; i < DEC_DB; ++i) o[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (int chunk = c_begin; chunk < c_end; ++chunk) {
    const int kb = chunk * DEC_KEYS;
    // (a page that holds no key the row sees may belong to nobody: one that does is read in its place, and masked)
    const bf16* pg[DEC_PAGES];
#pragma unroll
    for (int j = 0; j < DEC_PAGES; ++j) pg[j] = plane + (long)bt[min(max(chunk * DEC_PAGES + j, first_page), last_page)] * page_stride;
    const bf16* mine = plane + (long)bt[min(max(chunk * DEC_PAGES + wave, first_page), last_page)] * page_stride;
    bf16x8 k[DC];
#pragma unroll
    for (int dc = 0; dc < DC; ++dc) {
      const int d = dc * 32 + g * 8;
      k[dc] = d < KD ? *reinterpret_cast<const bf16x8*>(mine + (long)c16 * KD + d) : zero8;
    }
    bf16x4 v[DEC_DB][DEC_PAGES];
#pragma unroll
    for (int i = 0; i < DEC_DB; ++i) {
      const int db = min(wave + 4 * i, DB - 1);
#pragma unroll
      for (int j = 0; j < DEC_PAGES; ++j)
        v[i][j] = *reinterpret_cast<const bf16x4*>(pg[j] + (long)PAGE * KD + (long)(db * 16 + c16) * PAGE + 4 * g);
    }
    if (chunk == c_begin) {
#pragma unroll
      for (int j = 0; j < QN; ++j) {
        const int i = tid + j * 256, col = i / (KD / 8), piece = i % (KD / 8);
        if (i < 2 * KD) *reinterpret_cast<bf16x8*>(q_lds + col * DQ_STRIDE + piece * 8) = qreg[j];
      }
      __syncthreads();
    }
    f32x4 st0 = {0.f, 0.f, 0.f, 0.f}, st1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int dc = 0; dc < DC; ++dc) {
      const int d = dc * 32 + g * 8;
      const bf16x8 qv = d < KD ? *reinterpret_cast<const bf16x8*>(q_lds + c16 * DQ_STRIDE + d) : zero8;
      if (dc & 1) st1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[dc], qv, st1, 0, 0, 0);
      else st0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[dc], qv, st0, 0, 0, 0);
    }
    // the lane holds, for its column, the scores of the keys kb + 16 wave + 4g + i
    float sv[4], tmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key = kb + wave * PAGE + 4 * g + i;
      sv[i] = (key <= pos && key >= k_lo) ? (st0[i] + st1[i]) * scale_log2 : -INFINITY;
      tmax = fmaxf(tmax, sv[i]);
    }
    tmax = quad_max(tmax);
    if (g == 0) col_lds[wave][c16] = tmax;
    __syncthreads();
    const float m_new = fmaxf(fmaxf(fmaxf(col_lds[0][c16], col_lds[1][c16]), fmaxf(col_lds[2][c16], col_lds[3][c16])), m);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;           // no key yet: everything stays 0
    const float alpha = exp2f(m - m_use);
    bf16x4 p;
    float psum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float w = exp2f(sv[i] - m_use);
      psum += w;
      p[i] = static_cast<__bf16>(w);
    }
    p_lds[wave][lane] = p;
    l = l * alpha + psum;
    m = m_new;
    __syncthreads();
    const bool edge = kb + DEC_KEYS - 1 > pos || kb < k_lo;          // some of the slots lie outside what the row sees
    bf16x8 pb[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const bf16x4 lo = p_lds[2 * t][lane], hi = p_lds[2 * t + 1][lane];
      pb[t] = (bf16x8){lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
    }
#pragma unroll
    for (int i = 0; i < DEC_DB; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) o[i][e] *= alpha;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const bf16x4 lo = v[i][2 * t], hi = v[i][2 * t + 1];
        bf16x8 va = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
        if (edge) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int key0 = kb + 2 * t * PAGE + 4 * g + e, key1 = key0 + PAGE;
            if (key0 > pos || key0 < k_lo) va[e] = static_cast<__bf16>(0.f);
            if (key1 > pos || key1 < k_lo) va[4 + e] = static_cast<__bf16>(0.f);
          }
        }
        o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pb[t], o[i], 0, 0, 0);
      }
    }
  }
  // (a split without chunks leaves a maximum of -inf, a sum and results of zero)
  l = quad_sum(l);
  __syncthreads();
  if (g == 0) col_lds[wave][c16] = l;
  __syncthreads();
  const float lt = (col_lds[0][c16] + col_lds[1][c16]) + (col_lds[2][c16] + col_lds[3][c16]);
  if (head >= H) return;
  // the lane holds, for its column, the channels db * 16 + 4g + e of its wave's blocks
  const long slot = (row * H + head) * n_splits + split;
  const float inv = n_splits == 1 ? 1.f / (lt + sink_share(sinks, head, m)) : 1.f;
#pragma unroll
  for (int i = 0; i < DEC_DB; ++i) {
    const int db = wave + 4 * i;
    if (db >= DB) continue;
    if (n_splits == 1) {
      bf16x4 w;
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = static_cast<__bf16>(o[i][e] * inv);
      *reinterpret_cast<bf16x4*>(out + row * ldo + (long)head * VD + db * 16 + 4 * g) = w;
    } else {
      *reinterpret_cast<f32x4*>(part_o + slot * VD + db * 16 + 4 * g) = o[i];
    }
  }
  if (n_splits > 1 && g == 0 && wave == 0) part_ml[slot] = make_float2(m, lt);
}

// Portions of prompts: a workgroup of four waves takes an item of 64 columns (with fewer than 64 heads, 64 / heads
// consecutive rows of one request; else a row's heads in blocks of 64), 16 columns a wave. A step's keys and transposed
// values are copied into LDS once per workgroup and are every wave's MFMA operands from there, so a key is fetched
// once per 64 columns instead of once per 16. Key rows lie 16 bytes further apart in LDS than in memory, so that the
// sixteen keys a group of lanes reads at one channel offset fall into different banks.
static constexpr int TK_STRIDE = KD + 8;                       // elements between two keys in LDS
static constexpr int TK_BYTES = 32 * TK_STRIDE * 2, TV_BYTES = 2 * VD * PAGE * 2;

__global__ __launch_bounds__(256) void latent_tile_kernel(
    const bf16* __restrict__ q, long ldq, const bf16* __restrict__ plane, const int* __restrict__ block_tables, int bt_ld,
    const int* __restrict__ row_seq, const int* __restrict__ positions, const int2* __restrict__ items,
    bf16* __restrict__ out, long ldo, int H, float scale_log2, int window, const float* __restrict__ sinks) {
  __shared__ __attribute__((aligned(16))) bf16 k_lds[32 * TK_STRIDE];
  __shared__ __attribute__((aligned(16))) bf16 v_lds[2 * VD * PAGE];
  const int item = blockIdx.x, hb = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c16 = lane & 15, g = lane >> 4;
  const int row0 = items[item].x, n_rows = items[item].y;
  const int p_first = positions[row0];
  const int* bt = block_tables + (long)row_seq[row0] * bt_ld;
  const int p_last = p_first + n_rows - 1;
  const int c = wave * 16 + c16;                                // the lane's column among the item's 64
  const int ro = H >= 64 ? 0 : c / H;
  const int head = H >= 64 ? hb * 64 + c : c % H;
  const bool col_ok = ro < n_rows && head < H && (H >= 64 || c < (64 / H) * H);
  const int col_row = row0 + (col_ok ? ro : 0);
  const int col_pos = col_ok ? p_first + ro : -1;
  const int col_lo = window > 0 ? col_pos - window + 1 : 0;                // the column's first key
  const int k_lo = window > 0 ? max(0, p_first - window + 1) : 0;          // the first key any column sees
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};

  bf16x8 qb[DC];
#pragma unroll
  for (int dc = 0; dc < DC; ++dc) {
    const int d = dc * 32 + g * 8;
    qb[dc] = (col_ok && d < KD) ? *reinterpret_cast<const bf16x8*>(q + (long)col_row * ldq + (long)head * KD + d) : zero8;
  }
  f32x4 o[DB];
#pragma unroll
  for (int db = 0; db < DB; ++db) o[db] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const long page_stride = (long)PAGE * (KD + VD);
  const int s_first = k_lo / 32, n_steps = p_last / 32 + 1;     // (steps s_first .. n_steps - 1)
  constexpr int KP = KD / 8;                                    // 16-byte pieces of a key
  constexpr int VP = VD * PAGE / 8;                             // ... of a page's values

  // A thread's pieces of a step's keys and values, fetched into registers a step ahead (all loads issued together,
  // in flight while the step before is computed) and put into LDS between two barriers.
  constexpr int KN = (32 * KP + 255) / 256, VN = (2 * VP + 255) / 256;
  bf16x8 kreg[KN], vreg[VN];
  auto fetch = [&](int s) {
    const int kb = s * 32;
    const bool ok1 = kb + 16 <= p_last;
    const bf16* pg0 = plane + (long)bt[kb >> 4] * page_stride;
    const bf16* pg1 = plane + (long)(ok1 ? bt[(kb >> 4) + 1] : bt[kb >> 4]) * page_stride;
#pragma unroll
    for (int j = 0; j < KN; ++j) {
      const int i = tid + j * 256, key = i / KP, piece = i % KP;
      if (i < 32 * KP) kreg[j] = *reinterpret_cast<const bf16x8*>((key < 16 ? pg0 : pg1) + (long)(key & 15) * KD + piece * 8);
    }
#pragma unroll
    for (int j = 0; j < VN; ++j) {
      const int i = tid + j * 256, pgi = i / VP, piece = i % VP;
      if (i < 2 * VP) vreg[j] = *reinterpret_cast<const bf16x8*>((pgi ? pg1 : pg0) + (long)PAGE * KD + piece * 8);
    }
  };
  fetch(s_first);
  for (int s = s_first; s < n_steps; ++s) {
    const int kb = s * 32;
    const bool ok1 = kb + 16 <= p_last;
    __syncthreads();                                            // everyone has read the step before
#pragma unroll
    for (int j = 0; j < KN; ++j) {
      const int i = tid + j * 256, key = i / KP, piece = i % KP;
      if (i < 32 * KP) *reinterpret_cast<bf16x8*>(k_lds + key * TK_STRIDE + piece * 8) = kreg[j];
    }
#pragma unroll
    for (int j = 0; j < VN; ++j) {
      const int i = tid + j * 256;
      if (i < 2 * VP) *reinterpret_cast<bf16x8*>(v_lds + i * 8) = vreg[j];
    }
    __syncthreads();
    if (s + 1 < n_steps) fetch(s + 1);
    f32x4 st0 = {0.f, 0.f, 0.f, 0.f}, st1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int dc = 0; dc < DC; ++dc) {
      const int d = dc * 32 + g * 8;
      const bf16x8 k0 = d < KD ? *reinterpret_cast<const bf16x8*>(k_lds + c16 * TK_STRIDE + d) : zero8;
      const bf16x8 k1 = d < KD ? *reinterpret_cast<const bf16x8*>(k_lds + (16 + c16) * TK_STRIDE + d) : zero8;
      st0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0, qb[dc], st0, 0, 0, 0);
      st1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1, qb[dc], st1, 0, 0, 0);
    }
    float sv[8];
    float tmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int key0 = kb + 4 * g + i, key1 = key0 + 16;
      sv[i] = (key0 <= col_pos && key0 >= col_lo) ? st0[i] * scale_log2 : -INFINITY;
      sv[4 + i] = (ok1 && key1 <= col_pos && key1 >= col_lo) ? st1[i] * scale_log2 : -INFINITY;
      tmax = fmaxf(tmax, fmaxf(sv[i], sv[4 + i]));
    }
    tmax = quad_max(tmax);
    const float m_new = fmaxf(m, tmax);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = exp2f(m - m_use);
    float psum = 0.f;
    bf16x8 pb;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float p = exp2f(sv[e] - m_use);
      psum += p;
      pb[e] = static_cast<__bf16>(p);
    }
    l = l * alpha + psum;
    m = m_new;
    const bool edge = kb + 31 > p_last || kb < k_lo;
#pragma unroll
    for (int db = 0; db < DB; ++db) {
      const int off = (db * 16 + c16) * PAGE + 4 * g;
      const bf16x4 lo = *reinterpret_cast<const bf16x4*>(v_lds + off);
      const bf16x4 hi = ok1 ? *reinterpret_cast<const bf16x4*>(v_lds + VD * PAGE + off) : (bf16x4){0, 0, 0, 0};
      bf16x8 va = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
      if (edge) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key0 = kb + 4 * g + i, key1 = key0 + 16;
          if (key0 > p_last || key0 < k_lo) va[i] = static_cast<__bf16>(0.f);
          if (key1 > p_last || key1 < k_lo) va[4 + i] = static_cast<__bf16>(0.f);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) o[db][i] *= alpha;
      o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pb, o[db], 0, 0, 0);
    }
  }
  const float lt = quad_sum(l);
  if (!col_ok) return;
  const float inv = 1.f / (lt + sink_share(sinks, head, m));
  bf16* dst = out + (long)col_row * ldo + (long)head * VD + 4 * g;
#pragma unroll
  for (int db = 0; db < DB; ++db) {
    bf16x4 w;
#pragma unroll
    for (int i = 0; i < 4; ++i) w[i] = static_cast<__bf16>(o[db][i] * inv);
    *reinterpret_cast<bf16x4*>(dst + db * 16) = w;
  }
}

// The same items on eight waves, where two buffers of a step's keys and values fit into LDS. What bounds an item is what its
// workgroup reads from LDS, so the two products are cut differently: in the first a wave takes 16 columns and one of the
// step's two pages (keys are read once per 16 columns), in the second all 64 columns and every eighth block of 16 value
// channels (values are read once per workgroup; the weights, a sixteenth of their size, eight times). Keys and values go from
// the pages straight into LDS (no registers) a step ahead. Key rows lie an odd number of 16-byte pieces apart and a value
// channel's two pieces change places with every eighth channel, so that what sixteen lanes read at a time meets no bank
// conflict. A column's running maximum is raised only when a step exceeds it by 2^8 (weights then stay below 2^8), and
// sums are rescaled only in such steps. Sums run over the keys in order; a row's result does not depend on the item it is in.
static constexpr int T8_KPS = (KD / 8) | 1;                           // 16-byte pieces from one key to the next in LDS
static constexpr int T8_KI = (32 * T8_KPS + 63) / 64;                 // copies (64 pieces each) that bring a step's keys
static constexpr int T8_VI = (4 * VD + 63) / 64;                      // ... and its values
static constexpr int T8_LPW = (T8_KI + T8_VI + 7) / 8;                // copies a wave issues
static constexpr int T8_V_AT = T8_KI * 1024, T8_STAGE = T8_V_AT + T8_VI * 1024;      // bytes
static constexpr int T8_P_STRIDE = 80;                                // bytes from one column's weights to the next
static constexpr int T8_P_AT = 2 * T8_STAGE, T8_BYTES = T8_P_AT + 64 * T8_P_STRIDE + (2 + 1 + 2) * 64 * 4;
static constexpr bool T8_FITS = T8_BYTES <= 160 * 1024;
static constexpr int T8_DB = (DB + 7) / 8;                            // blocks of value channels a wave takes

#pragma clang diagnostic ignored "-Winline-asm"   // M0 in a clobber list: meant
// One 16-byte piece per lane from global memory straight into LDS, lane i's at lds_addr + 16 i; whoever reads the pieces
// waits for them (vmcnt) and for the other waves (barrier).
__device__ __forceinline__ void lt_copy16(const void* lane_src, unsigned lds_addr) {
  const unsigned base = (unsigned)__builtin_amdgcn_readfirstlane((int)lds_addr);
  asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off" : : "v"(lane_src), "s"(base) : "memory", "m0");
}

template <bool FITS>
__global__ __launch_bounds__(512) void latent_tile8_kernel(
    const bf16* __restrict__ q, long ldq, const bf16* __restrict__ plane, const int* __restrict__ block_tables, int bt_ld,
    const int* __restrict__ row_seq, const int* __restrict__ positions, const int2* __restrict__ items,
    bf16* __restrict__ out, long ldo, int H, float scale_log2, int window, const float* __restrict__ sinks) {
  __shared__ __attribute__((aligned(1024))) unsigned char lds[FITS ? T8_BYTES : 16];
  if (!FITS) return;
  const unsigned lds0 = (unsigned)(uintptr_t)(const __attribute__((address_space(3))) unsigned char*)lds;
  unsigned char* p_lds = lds + T8_P_AT;                               // [64 columns][32 keys] bfloat16
  float* max_lds = reinterpret_cast<float*>(p_lds + 64 * T8_P_STRIDE);      // [2 pages][64]: a step's maxima
  float* alpha_lds = max_lds + 128;                                   // [64]: what a column's sums are rescaled by
  float* sum_lds = alpha_lds + 64;                                    // [2][64]
  const int item = blockIdx.x, hb = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), c16 = lane & 15, g = lane >> 4;
  const int ct = wave & 3, kt = wave >> 2;                            // first product: the wave's 16 columns, its page
  const int row0 = items[item].x, n_rows = items[item].y;
  const int p_first = positions[row0], p_last = p_first + n_rows - 1;
  const int* bt = block_tables + (long)row_seq[row0] * bt_ld;
  // column c of the item: its row, its head, whether there is one
  auto row_of = [&](int c) { return H >= 64 ? 0 : c / H; };
  auto head_of = [&](int c) { return H >= 64 ? hb * 64 + c : c % H; };
  auto there = [&](int c) { return row_of(c) < n_rows && head_of(c) < H && (H >= 64 || c < (64 / H) * H); };
  const int c = ct * 16 + c16;
  const bool col_ok = there(c);
  const int col_pos = col_ok ? p_first + row_of(c) : -1;
  const int col_lo = window > 0 ? col_pos - window + 1 : 0;
  const int k_lo = window > 0 ? max(0, p_first - window + 1) : 0;     // the first key any column sees
  const int s_first = k_lo / 32, s_end = p_last / 32 + 1;
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const long page_bytes = (long)PAGE * (KD + VD) * 2;

  // the wave's copies: copy j = wave + 8 i brings 64 pieces of the buffer; a lane's piece by its page of the step (0, 1) and
  // its bytes from the page's start
  unsigned src_off[T8_LPW];
  bool src_second[T8_LPW];
#pragma unroll
  for (int i = 0; i < T8_LPW; ++i) {
    const int j = wave + 8 * i;
    if (j < T8_KI) {
      const int at = min(j * 64 + lane, 32 * T8_KPS - 1), key = at / T8_KPS, piece = min(at % T8_KPS, KD / 8 - 1);
      src_second[i] = key >= PAGE;
      src_off[i] = (unsigned)(((key & 15) * KD + piece * 8) * 2);
    } else {
      const int at = min((j - T8_KI) * 64 + lane, 4 * VD - 1), in_page = at % (2 * VD), ch = in_page >> 1;
      src_second[i] = at >= 2 * VD;
      src_off[i] = (unsigned)(PAGE * KD * 2 + ch * 32 + ((in_page & 1) ^ ((ch >> 3) & 1)) * 16);
    }
  }
  auto stage = [&](int s, int buf) {
    const int kb = s * 32;
    const unsigned char* pg0 = (const unsigned char*)plane + (long)bt[kb >> 4] * page_bytes;
    const unsigned char* pg1 = (const unsigned char*)plane + (long)bt[(kb >> 4) + (kb + 16 <= p_last ? 1 : 0)] * page_bytes;
#pragma unroll
    for (int i = 0; i < T8_LPW; ++i) {
      const int j = wave + 8 * i;
      if (j < T8_KI + T8_VI) lt_copy16((src_second[i] ? pg1 : pg0) + src_off[i], lds0 + buf * T8_STAGE + j * 1024);
    }
  };

  bf16x8 qb[DC];
#pragma unroll
  for (int dc = 0; dc < DC; ++dc) {
    const int d = dc * 32 + g * 8;
    qb[dc] = (col_ok && d < KD) ? *reinterpret_cast<const bf16x8*>(q + (long)(row0 + row_of(c)) * ldq + (long)head_of(c) * KD + d) : zero8;
  }
  f32x4 o[T8_DB][4];
#pragma unroll
  for (int i = 0; i < T8_DB; ++i)
#pragma unroll
    for (int t = 0; t < 4; ++t) o[i][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  stage(s_first, 0);
  for (int s = s_first; s < s_end; ++s) {
    const int kb = s * 32, buf = (s - s_first) & 1;
    asm volatile("s_waitcnt vmcnt(0)" : : : "memory");                // this wave's pieces of the step are in LDS
    __syncthreads();                                                  // ... and everyone's; everyone is done with the step before
    if (s + 1 < s_end) stage(s + 1, buf ^ 1);
    const unsigned char* st = lds + buf * T8_STAGE;
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int dc = 0; dc < DC; ++dc) {
      const int d = dc * 32 + g * 8;
      const bf16x8 k = d < KD ? *reinterpret_cast<const bf16x8*>(st + ((kt * 16 + c16) * T8_KPS + dc * 4 + g) * 16) : zero8;
      if (dc & 1) s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, qb[dc], s1, 0, 0, 0);
      else s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, qb[dc], s0, 0, 0, 0);
    }
    // the lane holds, for its column, the scores of the keys kb + 16 kt + 4g + i
    const bool edge = kb + 31 > p_first || kb < (window > 0 ? p_last - window + 1 : 0);      // some column does not see all of the step
    float sv[4], tmax = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sv[i] = (s0[i] + s1[i]) * scale_log2;
      if (edge) {
        const int key = kb + kt * 16 + 4 * g + i;
        sv[i] = (key <= col_pos && key >= col_lo) ? sv[i] : -INFINITY;
      }
      tmax = fmaxf(tmax, sv[i]);
    }
    tmax = quad_max(tmax);
    if (g == 0) max_lds[kt * 64 + c] = tmax;
    __syncthreads();
    const float step_max = fmaxf(max_lds[c], max_lds[64 + c]);
    const float m_new = step_max > m + 8.f ? step_max : m;            // (from -inf: the first step with a key)
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = m == m_new ? 1.f : exp2f(m - m_use);
    bf16x4 p;
    float psum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float w = exp2f(sv[i] - m_use);
      psum += w;
      p[i] = static_cast<__bf16>(w);
    }
    *reinterpret_cast<bf16x4*>(p_lds + c * T8_P_STRIDE + (kt * 16 + 4 * g) * 2) = p;
    if (kt == 0 && g == 0) alpha_lds[c] = alpha;
    l = l * alpha + psum;
    m = m_new;
    __syncthreads();
    // second product: lane (c16, g) brings the keys 8g .. 8g + 7 of the step for both operands
    bf16x8 pb[4];
    float al[4];
    bool rescale = false;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      pb[t] = *reinterpret_cast<const bf16x8*>(p_lds + (t * 16 + c16) * T8_P_STRIDE + g * 16);
      al[t] = alpha_lds[t * 16 + c16];
      rescale |= al[t] != 1.f;
    }
    if (__any(rescale)) {
#pragma unroll
      for (int i = 0; i < T8_DB; ++i)
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) o[i][t][e] *= al[t];
    }
    const bool outside = kb + 31 > p_last || kb < k_lo;               // some of the step's slots hold nothing any column sees
#pragma unroll
    for (int i = 0; i < T8_DB; ++i) {
      const int ch = min(wave + 8 * i, DB - 1) * 16 + c16;
      bf16x8 va = *reinterpret_cast<const bf16x8*>(st + T8_V_AT + ((g >> 1) * 2 * VD + ch * 2 + ((g & 1) ^ ((ch >> 3) & 1))) * 16);
      if (outside) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int key = kb + 8 * g + e;
          if (key > p_last || key < k_lo) va[e] = static_cast<__bf16>(0.f);
        }
      }
#pragma unroll
      for (int t = 0; t < 4; ++t) o[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pb[t], o[i][t], 0, 0, 0);
    }
  }
  l = quad_sum(l);
  __syncthreads();
  if (g == 0) sum_lds[kt * 64 + c] = l;
  if (kt == 0 && g == 0) max_lds[c] = m;
  __syncthreads();
  // the lane holds, for column t * 16 + c16, the channels db * 16 + 4g + e of its wave's blocks
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    const int cc = t * 16 + c16;
    if (!there(cc)) continue;
    const int head = head_of(cc);
    const float inv = 1.f / (sum_lds[cc] + sum_lds[64 + cc] + sink_share(sinks, head, max_lds[cc]));
    bf16* dst = out + (long)(row0 + row_of(cc)) * ldo + (long)head * VD + 4 * g;
#pragma unroll
    for (int i = 0; i < T8_DB; ++i) {
      const int db = wave + 8 * i;
      if (db >= DB) continue;
      bf16x4 w;
#pragma unroll
      for (int e = 0; e < 4; ++e) w[e] = static_cast<__bf16>(o[i][t][e] * inv);
      *reinterpret_cast<bf16x4*>(dst + db * 16) = w;
    }
  }
}

// out[row, head, :] = sum_s 2^(m_s - M) o_s / sum_s 2^(m_s - M) l_s over a (row, head)'s splits, in a fixed order
__global__ __launch_bounds__(256) void latent_merge_kernel(const float* __restrict__ part_o, const float2* __restrict__ part_ml,
                                                           bf16* __restrict__ out, long ldo, int H, int n_splits,
                                                           const float* __restrict__ sinks) {
  __shared__ float w[256];                 // the weights of up to 256 splits at a time
  __shared__ float red[16];
  const long row = blockIdx.x;
  const int head = blockIdx.y, t = threadIdx.x;
  const long base = (row * H + head) * n_splits;
  float M = -INFINITY;
  for (int s = t; s < n_splits; s += 256) M = fmaxf(M, part_ml[base + s].x);
  M = block_max(M, red);
  float L = 0.f;
  float acc[(VD + 255) / 256];
#pragma unroll
  for (int j = 0; j < (VD + 255) / 256; ++j) acc[j] = 0.f;
  for (int s0 = 0; s0 < n_splits; s0 += 256) {
    const int cnt = min(256, n_splits - s0);
    float mine = 0.f, share = 0.f;
    if (t < cnt) {
      const float2 ml = part_ml[base + s0 + t];
      if (ml.x != -INFINITY) {             // else: a split that held no key of this row (its partial output is zero)
        mine = exp2f(ml.x - M);
        share = mine * ml.y;
      }
    }
    __syncthreads();
    w[t] = mine;
    L += block_sum(share, red);            // its barriers also publish w[]
    // (a split's partial outputs are independent loads: several are in flight at a time)
#pragma unroll
    for (int j = 0; j < (VD + 255) / 256; ++j) {
      const int c = j * 256 + t;
      if (c >= VD) continue;
      const float* src = part_o + (base + s0) * VD + c;
      float a = 0.f;
#pragma unroll 8
      for (int s = 0; s < cnt; ++s) a += w[s] * src[(long)s * VD];
      acc[j] += a;
    }
  }
  L += sink_share(sinks, head, M);         // the sink's share of the denominator, once for all splits
#pragma unroll
  for (int j = 0; j < (VD + 255) / 256; ++j) {
    const int c = j * 256 + t;
    if (c < VD) out[row * ldo + (long)head * VD + c] = static_cast<__bf16>(acc[j] / L);
  }
}

TIS_EXPORT int tis_attention_latent_dims() { return TIS_LATENT; }

// items: (first row, rows) per item of the kernel for portions (64 columns each: 64 / H rows, or a row's heads in blocks of
// 64), which takes every item's keys whole (n_splits 0). Null: `rows` single rows, whose keys are cut into n_splits parts;
// part_o / part_ml: [rows][H][n_splits][VD] floats and [rows][H][n_splits] (maximum, sum) pairs where n_splits > 1.
TIS_EXPORT int tis_attention_latent(const void* q, long ldq, const void* plane, const int* block_tables, int bt_ld,
                                    const int* row_seq, const int* positions, const int* items, int n_items, void* out,
                                    long ldo, float* part_o, float* part_ml, int rows, int H, int key_dim, int value_dim,
                                    int page_size, float scale, int n_splits, int window, const float* sinks, hipStream_t stream) {
  if (rows == 0 || n_items == 0) return 0;
  if (key_dim != KD || value_dim != VD) return tis_fail("attention_latent: built for keys of %d and values of %d, called with %d and %d", KD, VD, key_dim, value_dim);
  if (page_size != PAGE) return tis_fail("attention_latent: pages of %d slots (this kernel takes %d)", page_size, PAGE);
  if (rows < 0 || n_items < 0 || H < 1 || window < 0 || n_splits < 0 || n_splits > 65535 || (H + 15) / 16 > 65535)
    return tis_fail("attention_latent: bad size rows=%d items=%d heads=%d splits=%d", rows, n_items, H, n_splits);
  if (n_splits > 1 && (!part_o || !part_ml)) return tis_fail("attention_latent: %d splits need a workspace", n_splits);
  if ((ldq % 8) || (ldo % 4) || ((uintptr_t)q % 16) || ((uintptr_t)out % 8) || ((uintptr_t)plane % 16))
    return tis_fail("attention_latent: q, out and the cache plane must be 16-byte aligned with row strides in steps of 8");
  if (n_splits == 0) {
    if (!items) return tis_fail("attention_latent: the four-wave kernel needs its list of items");
    dim3 tgrid(n_items, (H + 63) / 64);
    if (T8_FITS) {
      latent_tile8_kernel<T8_FITS><<<tgrid, 512, 0, stream>>>((const bf16*)q, ldq, (const bf16*)plane, block_tables, bt_ld, row_seq,
                                                             positions, (const int2*)items, (bf16*)out, ldo, H,
                                                             scale * 1.4426950408889634f, window, sinks);
      return tis_launch_status("attention_latent tiles");
    }
    latent_tile_kernel<<<tgrid, 256, 0, stream>>>((const bf16*)q, ldq, (const bf16*)plane, block_tables, bt_ld, row_seq,
                                                  positions, (const int2*)items, (bf16*)out, ldo, H,
                                                  scale * 1.4426950408889634f, window, sinks);
    return tis_launch_status("attention_latent tiles");
  }
  if (items || n_items != rows) return tis_fail("attention_latent: single rows come without a list (%d items of %d rows)", n_items, rows);
  dim3 grid(rows, (H + 15) / 16, n_splits);
  latent_decode_kernel<<<grid, 256, 0, stream>>>((const bf16*)q, ldq, (const bf16*)plane, block_tables, bt_ld, row_seq, positions,
                                                (bf16*)out, ldo, part_o, (float2*)part_ml, H, scale * 1.4426950408889634f,
                                                n_splits, window, sinks);
  int rc = tis_launch_status("attention_latent");
  if (rc || n_splits == 1) return rc;
  dim3 mgrid(rows, H);
  latent_merge_kernel<<<mgrid, 256, 0, stream>>>(part_o, (const float2*)part_ml, (bf16*)out, ldo, H, n_splits, sinks);
  return tis_launch_status("attention_latent merge");
}
