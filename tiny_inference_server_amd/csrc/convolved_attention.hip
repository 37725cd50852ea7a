// Around an attention whose queries, keys and values pass a short convolution and whose values are turned by their
// position: the step before it (bias, convolution, rotation, pages, the convolution's state), and the turn back of its
// results where the attention kernel has not done that itself.
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
  int rows, C, K, H, G, KD, VD, page_size, chunk;
};

// grid (chunks of rows, H + 2 G), one wave each: unit u < H is a query head, u < H + G a key head, else a value head. A
// lane owns pairs of channels and walks the chunk's rows with the last taps - 1 rows in registers (KT taps; KT 0: any
// number, read again from memory). The rows of a request that reach into its state line are all done by the wave that has
// the request's first row, which writes the line behind the last of them: nobody else looks at it.
template <typename T, int KT>
__global__ __launch_bounds__(TIS_WAVE) void convolved_prepare_kernel(ConvolvedArgs a, T* __restrict__ plane,
                                                                     T* __restrict__ q_out, long ldq) {
  const int K = KT ? KT : a.K;
  constexpr int KW = KT > 1 ? KT - 1 : 1;
  const int u = blockIdx.y, lane = threadIdx.x;
  const bool is_q = u < a.H, is_k = !is_q && u < a.H + a.G;
  const int head = is_q ? u : is_k ? u - a.H : u - a.H - a.G;
  const int dim = is_q || is_k ? a.KD : a.VD;
  const int base = is_q ? head * a.KD : is_k ? (a.H + head) * a.KD : (a.H + a.G) * a.KD + head * a.VD;
  const int rot = is_q || is_k ? a.rot_dims : (a.turn_freqs ? a.VD : 0);
  const float* freqs = is_q || is_k ? a.freqs : a.turn_freqs;
  const float factor = is_q || is_k ? a.rot_factor : 1.f;
  const long page_stride = (long)a.G * a.page_size * (a.KD + a.VD);

  // the first row of the chunk that is this wave's to do
  long begin = (long)blockIdx.x * a.chunk;
  const long end = min(begin + a.chunk, (long)a.rows);
  {
    const int seq = a.row_seq[begin], first = a.cu_rows[seq], n = a.cu_rows[seq + 1] - first;
    const int t = (int)(begin - first);
    if (t > 0 && t < K - 1) begin = first + min(n, K - 1);
  }
  if (begin >= end) return;

  for (int p = lane; 2 * p < dim; p += TIS_WAVE) {
    const int c = base + 2 * p;
    const bool two = 2 * p + 1 < dim;
    const float b0 = a.bias[c], b1 = two ? a.bias[c + 1] : 0.f;
    const bool turns = 2 * p + 1 < rot;
    const float freq = turns ? freqs[p] : 0.f;
    auto raw = [&](long row) {
      const float* s = a.proj + row * a.ldp + c;
      return make_float2(s[0] + b0, two ? s[1] + b1 : 0.f);
    };
    float w0[KT ? KT : 1], w1[KT ? KT : 1];
    if (KT) {
#pragma unroll
      for (int j = 0; j < KT; ++j) {
        w0[j] = a.taps[(long)c * K + j];
        w1[j] = two ? a.taps[(long)(c + 1) * K + j] : 0.f;
      }
    }
    float2 win[KW];
    bool have = false;
    long limit = end;
    for (long r = begin; r < limit; ++r) {
      const int seq = a.row_seq[r], first = a.cu_rows[seq], n = a.cu_rows[seq + 1] - first;
      const int t = (int)(r - first);
      float* line = K > 1 ? a.state + (long)a.seq_slots[seq] * a.state_ld + c : nullptr;
      auto kept = [&](int k) { return make_float2(line[(long)k * a.C], two ? line[(long)k * a.C + 1] : 0.f); };
      if (t == 0) {
        limit = max(limit, (long)first + min(n, K - 1));
        if (KT > 1) {
#pragma unroll
          for (int k = 0; k < KW; ++k) win[k] = kept(k);
          have = true;
        }
      } else if (KT > 1 && !have) {
#pragma unroll
        for (int k = 0; k < KW; ++k) win[k] = raw(r - KW + k);       // (t >= K - 1 here: see `begin`)
        have = true;
      }
      const float2 now = raw(r);
      float x = 0.f, y = 0.f;
      if (KT) {
#pragma unroll
        for (int k = 0; k < KT - 1; ++k) {
          x += w0[k] * win[k].x;
          y += w1[k] * win[k].y;
        }
        x += w0[KT - 1] * now.x;
        y += w1[KT - 1] * now.y;
#pragma unroll
        for (int k = 0; k + 1 < KT - 1; ++k) win[k] = win[k + 1];
        if (KT > 1) win[KW - 1] = now;
      } else {
        for (int j = 0; j < K; ++j) {
          const int back = K - 1 - j;
          const float2 v = back <= t ? raw(r - back) : kept(K - 1 + t - back);
          x += a.taps[(long)c * K + j] * v.x;
          if (two) y += a.taps[(long)(c + 1) * K + j] * v.y;
        }
      }
      if (K > 1 && t == min(n, K - 1) - 1) {
        // the last of the rows that read the line: entry k becomes the step's row n - (K - 1) + k, or an older entry (in
        // rising order: an entry that is still to be read has not been written)
        for (int k = 0; k < K - 1; ++k) {
          const int at = n - (K - 1) + k;
          const float2 v = at >= 0 ? raw(first + at) : kept(k + n);
          line[(long)k * a.C] = v.x;
          if (two) line[(long)k * a.C + 1] = v.y;
        }
      }
      if (turns) {
        float sn, cs;
        sincosf((float)a.positions[r] * freq, &sn, &cs);
        if (!is_q && !is_k && head == 0 && a.turn) a.turn[r * (a.VD / 2) + p] = make_float2(cs, sn);
        sn *= factor;
        cs *= factor;
        const float rx = x * cs - y * sn, ry = y * cs + x * sn;
        x = rx;
        y = ry;
      }
      if (is_q) {
        T* dst = q_out + r * ldq + (long)head * a.KD + 2 * p;
        dst[0] = from_f<T>(x);
        if (two) dst[1] = from_f<T>(y);
        continue;
      }
      const int ws = a.write_slots[r];
      T* page = plane + (long)(ws / a.page_size) * page_stride;
      const int slot = ws % a.page_size;
      if (is_k) {
        T* dst = page + ((long)head * a.page_size + slot) * a.KD + 2 * p;
        dst[0] = from_f<T>(x);
        if (two) dst[1] = from_f<T>(y);
      } else {
        T* dst = page + (long)a.G * a.page_size * a.KD + ((long)head * a.VD + 2 * p) * a.page_size + slot;
        dst[0] = from_f<T>(x);
        if (two) dst[a.page_size] = from_f<T>(y);
      }
    }
  }
}

// In place: every head's pairs (2m, 2m + 1) of a row are turned back by the angle whose (cos, sin) is turn[row][m].
template <typename T>
__global__ __launch_bounds__(256) void turn_back_kernel(T* __restrict__ x, long ldx, const float2* __restrict__ turn, long rows,
                                                        int H, int V) {
  const int half = V / 2;
  const long i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * H * half) return;
  const long r = i / ((long)H * half);
  const int j = (int)(i % ((long)H * half));
  const float2 cs = turn[r * half + j % half];
  T* p = x + r * ldx + (long)(j / half) * V + 2 * (j % half);
  const float a = to_f(p[0]), b = to_f(p[1]);
  p[0] = from_f<T>(a * cs.x + b * cs.y);
  p[1] = from_f<T>(b * cs.x - a * cs.y);
}

TIS_EXPORT int tis_convolved_prepare(int dtype, const float* proj, long ldp, const float* bias, const float* taps, float* state,
                                     long state_ld, const int* row_seq, const int* cu_rows, const int* seq_slots,
                                     const int* positions, const int* write_slots, void* plane, void* q_out, long ldq,
                                     const float* freqs, int rot_dims, float rot_factor, const float* turn_freqs, float* turn,
                                     int rows, int K, int H, int G, int KD, int VD, int page_size, int chunk,
                                     hipStream_t stream) {
  if (rows == 0) return 0;
  const long C = (long)H * KD + (long)G * (KD + VD);
  if (rows < 0 || H < 1 || G < 1 || H % G || KD < 1 || VD < 1 || page_size < 1 || chunk < 1 || H + 2 * G > 65535 || C > (1 << 24))
    return tis_fail("convolved_prepare: bad size rows=%d heads=%d kv_heads=%d key=%d value=%d page=%d", rows, H, G, KD, VD, page_size);
  if (K < 1 || K > CV_MAX_TAPS) return tis_fail("convolved_prepare: %d taps (1 to %d)", K, CV_MAX_TAPS);
  if (K > 1 && (!state || state_ld < (long)(K - 1) * C))
    return tis_fail("convolved_prepare: state lines of %ld floats for %ld", state_ld, (long)(K - 1) * C);
  if (rot_dims < 0 || rot_dims > KD || rot_dims % 2 || (rot_dims && !freqs))
    return tis_fail("convolved_prepare: %d rotated channels of %d", rot_dims, KD);
  if (turn_freqs && (VD % 2 || !turn)) return tis_fail("convolved_prepare: values of %d channels turn in pairs, with room for their angles", VD);
  if (!proj || !bias || !taps || !write_slots || !plane || !q_out) return tis_fail("convolved_prepare: a pointer is missing");
  const ConvolvedArgs a{proj, ldp, bias, taps, state, state_ld, row_seq, cu_rows, seq_slots, positions, write_slots, freqs,
                        rot_dims, rot_factor, turn_freqs, (float2*)turn, rows, (int)C, K, H, G, KD, VD, page_size, chunk};
  dim3 grid((rows + chunk - 1) / chunk, H + 2 * G);
#define CV_LAUNCH(T, KT) convolved_prepare_kernel<T, KT><<<grid, TIS_WAVE, 0, stream>>>(a, (T*)plane, (T*)q_out, ldq)
#define CV_BY_TAPS(T)                  \
  if (K == 1) CV_LAUNCH(T, 1);         \
  else if (K == 2) CV_LAUNCH(T, 2);    \
  else if (K == 3) CV_LAUNCH(T, 3);    \
  else if (K == 4) CV_LAUNCH(T, 4);    \
  else CV_LAUNCH(T, 0);
  if (dtype == TIS_F32) { CV_BY_TAPS(float) }
  else if (dtype == TIS_BF16) { CV_BY_TAPS(bf16) }
  else return tis_fail("unknown dtype code %d", dtype);
#undef CV_BY_TAPS
#undef CV_LAUNCH
  return tis_launch_status("convolved_prepare");
}

TIS_EXPORT int tis_turn_back(int dtype, void* x, long ldx, const float* turn, int rows, int H, int V, hipStream_t stream) {
  if (rows == 0) return 0;
  if (rows < 0 || H < 1 || V < 2 || V % 2 || !turn) return tis_fail("turn_back: bad size rows=%d heads=%d channels=%d", rows, H, V);
  const long blocks = ((long)rows * H * (V / 2) + 255) / 256;
  if (dtype == TIS_F32) turn_back_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, ldx, (const float2*)turn, rows, H, V);
  else if (dtype == TIS_BF16) turn_back_kernel<bf16><<<blocks, 256, 0, stream>>>((bf16*)x, ldx, (const float2*)turn, rows, H, V);
  else return tis_fail("unknown dtype code %d", dtype);
  return tis_launch_status("turn_back");
}
