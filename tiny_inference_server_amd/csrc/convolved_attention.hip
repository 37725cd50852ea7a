// The step before an attention whose queries, keys and values pass a short convolution and whose values are turned by
// their position: bias, convolution, rotation, pages, the convolution's state. (The attention kernels turn their results
// back.)
//
// A request's state line is [taps - 1][channels] 32-bit floats, the last projected rows (with their bias), oldest first; a
// line taken anew is all zeros, which is what lies before a sequence's first row. A row reads the rows before it from this
// step's rows where they are part of the step and from the line otherwise, so a result does not depend on where a prompt
// was cut. Everything is 32-bit; `T` is the type of queries and pages.
#include "common.h"

TIS_DEFINE_LAST_ERROR(tis_convolved)

static constexpr int CV_MAX_TAPS = 64;

struct ConvolvedArgs {
  const float* proj;        // [rows][ldp]: queries of all heads, keys, values side by side
  long ldp;
  const float* bias;        // [channels]
  const float* taps;        // [channels][K], the last one weighs the row itself
  float* state;             // lines of state_ld floats; null with one tap
  long state_ld;
  const int* row_seq;
  const int* cu_rows;
  const int* seq_slots;
  const int* positions;
  const int* write_slots;
  const float* freqs;       // [rot_dims / 2]: angle = position * freqs[pair] of queries and keys, pairs (2i, 2i + 1)
  int rot_dims;
  float rot_factor;         // on cosine and sine
  const float* turn_freqs;  // [VD / 2]: the same for values, or null: values stay
  float2* turn;             // [rows][VD / 2]: (cos, sin) of the values' angles, for the turn back
  int rows, C, K, H, G, KD, VD, page_size;
};

static constexpr int CV_ROWS = 8;      // rows of a chunk where rows are many

// A row of the chunk as its workgroup needs it.
struct ConvolvedRow {
  int t, n;              // which of its request's rows of this step it is, and of how many
  int slot;              // the request's state line
  int pos, ws;           // position, slot in the pages
};

template <typename T> struct alignas(16) RowRun { T v[CV_ROWS]; };           // eight slots' values of a channel, stored whole
template <typename T> struct alignas(2 * sizeof(T)) Pair { T v[2]; };

// grid (chunks of `chunk` rows, blocks of four units), four waves a workgroup, a unit each: unit u < H is a query head, u < H +
// G a key head, else a value head. The rows' angles are worked out once per workgroup, into LDS. A lane owns pairs of
// channels. The rows of a request that reach into its state line are all done by the workgroup that has the request's first
// row (beyond its chunk's end where need be), and the line is written back by the wave that has read it: nobody else looks
// at it. KT: taps (0: any number). EVEN: pairs are whole and aligned everywhere.
template <typename T, int KT, bool EVEN>
__global__ __launch_bounds__(256) void convolved_prepare_kernel(ConvolvedArgs a, T* __restrict__ plane, T* __restrict__ q_out,
                                                                long ldq, int chunk) {
  extern __shared__ float2 cv_lds[];
  const int K = KT ? KT : a.K;
  const int tid = threadIdx.x, lane = tid & 63;
  const long page_stride = (long)a.G * a.page_size * (a.KD + a.VD);
  const int half_q = a.rot_dims / 2, half_v = a.turn_freqs ? a.VD / 2 : 0;

  // the rows this workgroup does: from the first of the chunk that reaches into nobody else's line ...
  long begin = (long)blockIdx.x * chunk;
  const long end = min(begin + chunk, (long)a.rows);
  {
    const int seq = a.row_seq[begin], first = a.cu_rows[seq], n = a.cu_rows[seq + 1] - first;
    const int t = (int)(begin - first);
    if (t > 0 && t < K - 1) begin = first + min(n, K - 1);
  }
  if (begin >= end) return;
  // ... to the chunk's end, or to the last row that reaches into the line of a request that begins in the chunk
  long limit = end;
  {
    const int seq = a.row_seq[end - 1], first = a.cu_rows[seq], n = a.cu_rows[seq + 1] - first;
    if (first >= begin) limit = max(end, (long)first + min(n, K - 1));
  }
  const int n_rows = (int)(limit - begin);
  float2* ang_q = cv_lds;
  float2* ang_v = ang_q + (long)(chunk + K - 1) * half_q;
  ConvolvedRow* meta = reinterpret_cast<ConvolvedRow*>(ang_v + (long)(chunk + K - 1) * half_v);
  for (int i = tid; i < n_rows; i += 256) {
    const int seq = a.row_seq[begin + i], first = a.cu_rows[seq];
    meta[i] = ConvolvedRow{(int)(begin + i - first), a.cu_rows[seq + 1] - first, a.seq_slots[seq], a.positions[begin + i],
                           a.write_slots[begin + i]};
  }
  for (int i = tid; i < n_rows * (half_q + half_v); i += 256) {
    const int r = i / (half_q + half_v), p = i % (half_q + half_v);
    const float pos = (float)a.positions[begin + r];
    float sn, cs;
    if (p < half_q) {
      sincosf(pos * a.freqs[p], &sn, &cs);
      ang_q[r * half_q + p] = make_float2(cs * a.rot_factor, sn * a.rot_factor);
    } else {
      sincosf(pos * a.turn_freqs[p - half_q], &sn, &cs);
      ang_v[r * half_v + p - half_q] = make_float2(cs, sn);
      if (blockIdx.y == 0 && a.turn) a.turn[(begin + r) * half_v + p - half_q] = make_float2(cs, sn);
    }
  }
  __syncthreads();

  const int u = blockIdx.y * 4 + (tid >> 6);
  if (u >= a.H + 2 * a.G) return;
  const bool is_q = u < a.H, is_k = !is_q && u < a.H + a.G, is_v = !is_q && !is_k;
  const int head = is_q ? u : is_k ? u - a.H : u - a.H - a.G;
  const int dim = is_v ? a.VD : a.KD;
  const int base = is_q ? head * a.KD : is_k ? (a.H + head) * a.KD : (a.H + a.G) * a.KD + head * a.VD;
  const int half = is_v ? half_v : half_q;
  const float2* ang = is_v ? ang_v : ang_q;
  auto turned = [&](float2 v, int i, int p) {
    if (p >= half) return v;
    const float2 cs = ang[i * half + p];
    return make_float2(v.x * cs.x - v.y * cs.y, v.y * cs.x + v.x * cs.y);
  };
  auto value_at = [&](int ws, int p) {                  // the first of the pair's channels in the page of slot ws
    return plane + (long)(ws / a.page_size) * page_stride + (long)a.G * a.page_size * a.KD +
           ((long)head * a.VD + 2 * p) * a.page_size + ws % a.page_size;
  };

  // eight rows of one request, none of which reaches into its line, in eight slots that follow one another: straight through,
  // everything asked for at once
  if (KT && EVEN && n_rows == CV_ROWS && meta[0].t >= K - 1 && meta[CV_ROWS - 1].t == meta[0].t + CV_ROWS - 1 &&
      a.page_size % CV_ROWS == 0 && meta[0].ws % CV_ROWS == 0) {
    constexpr int KW = KT ? KT : 1;
    const int ws = meta[0].ws;
    for (int p = lane; 2 * p < dim; p += TIS_WAVE) {
      const int c = base + 2 * p;
      const float2 bias = *reinterpret_cast<const float2*>(a.bias + c);
      float2 in[CV_ROWS + KW - 1];
#pragma unroll
      for (int i = 0; i < CV_ROWS + KW - 1; ++i)
        in[i] = *reinterpret_cast<const float2*>(a.proj + (begin + i - (KW - 1)) * a.ldp + c);
      float w0[KW], w1[KW];
#pragma unroll
      for (int j = 0; j < KW; ++j) {
        w0[j] = a.taps[(long)c * KW + j];
        w1[j] = a.taps[(long)(c + 1) * KW + j];
      }
#pragma unroll
      for (int i = 0; i < CV_ROWS + KW - 1; ++i) {
        in[i].x += bias.x;
        in[i].y += bias.y;
      }
      RowRun<T> v0, v1;
#pragma unroll
      for (int i = 0; i < CV_ROWS; ++i) {
        float2 v = make_float2(0.f, 0.f);
#pragma unroll
        for (int j = 0; j < KW; ++j) {
          v.x += w0[j] * in[i + j].x;
          v.y += w1[j] * in[i + j].y;
        }
        v = turned(v, i, p);
        v0.v[i] = from_f<T>(v.x);
        v1.v[i] = from_f<T>(v.y);
      }
      if (is_v) {
        T* dst = value_at(ws, p);
        *reinterpret_cast<RowRun<T>*>(dst) = v0;
        *reinterpret_cast<RowRun<T>*>(dst + a.page_size) = v1;
      } else {
        T* dst = is_q ? q_out + begin * ldq + (long)head * a.KD + 2 * p
                      : plane + (long)(ws / a.page_size) * page_stride + ((long)head * a.page_size + ws % a.page_size) * a.KD + 2 * p;
        const long step = is_q ? ldq : a.KD;
#pragma unroll
        for (int i = 0; i < CV_ROWS; ++i) *reinterpret_cast<Pair<T>*>(dst + i * step) = Pair<T>{{v0.v[i], v1.v[i]}};
      }
    }
    return;
  }

  for (int p = lane; 2 * p < dim; p += TIS_WAVE) {
    const int c = base + 2 * p;
    const bool two = EVEN || 2 * p + 1 < dim;
    const int c1 = two ? c + 1 : c;
    const float b0 = a.bias[c], b1 = a.bias[c1];
#pragma unroll 4
    for (int i = 0; i < n_rows; ++i) {
      const long r = begin + i;
      const ConvolvedRow m = meta[i];
      const float* line = K > 1 ? a.state + (long)m.slot * a.state_ld : nullptr;
      // the channels' numbers `back` rows before this one, from the step's rows or from the line
      auto before = [&](int back) {
        const bool here = back <= m.t;
        const float* s = here ? a.proj + (r - back) * a.ldp : line + (long)(K - 1 + m.t - back) * a.C;
        return make_float2(s[c] + (here ? b0 : 0.f), s[c1] + (here ? b1 : 0.f));
      };
      float2 v = make_float2(0.f, 0.f);
#pragma unroll 4
      for (int j = 0; j < K; ++j) {
        const float2 in = before(K - 1 - j);
        v.x += a.taps[(long)c * K + j] * in.x;
        v.y += a.taps[(long)c1 * K + j] * in.y;
      }
      v = turned(v, i, p);
      T* dst;
      long step = 1;
      if (is_q) {
        dst = q_out + r * ldq + (long)head * a.KD + 2 * p;
      } else if (is_k) {
        dst = plane + (long)(m.ws / a.page_size) * page_stride + ((long)head * a.page_size + m.ws % a.page_size) * a.KD + 2 * p;
      } else {
        dst = value_at(m.ws, p);
        step = a.page_size;
      }
      dst[0] = from_f<T>(v.x);
      if (two) dst[step] = from_f<T>(v.y);
    }
    // the lines of the requests that begin here, now that their readers are done: entry k becomes the step's row
    // n - (K - 1) + k, or an older entry (in rising order: an entry that is still to be read has not been written)
    for (int i = 0; i < n_rows && K > 1; ++i) {
      const ConvolvedRow m = meta[i];
      if (m.t) continue;
      float* line = a.state + (long)m.slot * a.state_ld;
      const float* first = a.proj + (begin + i) * a.ldp;
      for (int k = 0; k < K - 1; ++k) {
        const int at = m.n - (K - 1) + k;
        const float* s = at >= 0 ? first + at * a.ldp : line + (long)(k + m.n) * a.C;
        const float x = s[c] + (at >= 0 ? b0 : 0.f), y = s[c1] + (at >= 0 ? b1 : 0.f);
        line[(long)k * a.C + c] = x;
        line[(long)k * a.C + c1] = two ? y : x;
      }
    }
  }
}

TIS_EXPORT int tis_convolved_prepare(int dtype, const float* proj, long ldp, const float* bias, const float* taps, float* state,
                                     long state_ld, const int* row_seq, const int* cu_rows, const int* seq_slots,
                                     const int* positions, const int* write_slots, void* plane, void* q_out, long ldq,
                                     const float* freqs, int rot_dims, float rot_factor, const float* turn_freqs, float* turn,
                                     int rows, int K, int H, int G, int KD, int VD, int page_size, hipStream_t stream) {
  if (rows == 0) return 0;
  const long C = (long)H * KD + (long)G * (KD + VD);
  if (rows < 0 || H < 1 || G < 1 || H % G || KD < 1 || VD < 1 || page_size < 1 || H + 2 * G > 65535 || C > (1 << 24))
    return tis_fail("convolved_prepare: bad size rows=%d heads=%d kv_heads=%d key=%d value=%d page=%d", rows, H, G, KD, VD, page_size);
  if (K < 1 || K > CV_MAX_TAPS) return tis_fail("convolved_prepare: %d taps (1 to %d)", K, CV_MAX_TAPS);
  if (K > 1 && (!state || state_ld < (long)(K - 1) * C))
    return tis_fail("convolved_prepare: state lines of %ld floats for %ld", state_ld, (long)(K - 1) * C);
  if (rot_dims < 0 || rot_dims > KD || rot_dims % 2 || (rot_dims && !freqs))
    return tis_fail("convolved_prepare: %d rotated channels of %d", rot_dims, KD);
  if (turn_freqs && (VD % 2 || !turn)) return tis_fail("convolved_prepare: values of %d channels turn in pairs, with room for their angles", VD);
  if (!proj || !bias || !taps || !write_slots || !plane || !q_out) return tis_fail("convolved_prepare: a pointer is missing");
  const ConvolvedArgs a{proj, ldp, bias, taps, state, state_ld, row_seq, cu_rows, seq_slots, positions, write_slots, freqs,
                        rot_dims, rot_factor, turn_freqs, (float2*)turn, rows, (int)C, K, H, G, KD, VD, page_size};
  // few rows: one a workgroup, so that a step still fills the chip; many: eight, as long as their angles fit into LDS
  const long per_row = (long)(rot_dims / 2 + (turn_freqs ? VD / 2 : 0)) * sizeof(float2) + sizeof(ConvolvedRow);
  const int chunk = rows > 256 && (CV_ROWS + K - 1) * per_row <= 48 * 1024 ? CV_ROWS : 1;
  const long lds = (chunk + K - 1) * per_row;
  if (lds > 64 * 1024) return tis_fail("convolved_prepare: %ld bytes of angles for %d taps and heads of %d and %d", lds, K, KD, VD);
  const bool even = KD % 2 == 0 && VD % 2 == 0 && ldp % 2 == 0 && ldq % 2 == 0 &&
                    (((uintptr_t)proj | (uintptr_t)bias) % 8) == 0 && (((uintptr_t)plane | (uintptr_t)q_out) % 16) == 0;
  dim3 grid((rows + chunk - 1) / chunk, (H + 2 * G + 3) / 4);
#define CV_LAUNCH(T, KT)                                                                                            \
  if (even) convolved_prepare_kernel<T, KT, true><<<grid, 256, lds, stream>>>(a, (T*)plane, (T*)q_out, ldq, chunk); \
  else convolved_prepare_kernel<T, KT, false><<<grid, 256, lds, stream>>>(a, (T*)plane, (T*)q_out, ldq, chunk)
#define CV_BY_TAPS(T)                  \
  if (K == 2) { CV_LAUNCH(T, 2); }     \
  else if (K == 3) { CV_LAUNCH(T, 3); } \
  else if (K == 4) { CV_LAUNCH(T, 4); } \
  else { CV_LAUNCH(T, 0); }
  if (dtype == TIS_F32) { CV_BY_TAPS(float) }
  else if (dtype == TIS_BF16) { CV_BY_TAPS(bf16) }
  else return tis_fail("unknown dtype code %d", dtype);
#undef CV_BY_TAPS
#undef CV_LAUNCH
  return tis_launch_status("convolved_prepare");
}
