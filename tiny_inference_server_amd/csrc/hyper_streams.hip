// A residual of S streams in 32-bit: the end of one sublayer and the beginning of the next in one pass over a row.
//
//   X_t <- sum_s mix[s][t] X_s + out[t] (y + bias)     every new stream from all the old ones (y null: X stays as it is)
//   u = sum_t read[t] X_t;  h = u / sqrt(mean(u^2) + eps) * gain
//   h' = h + (h_before - h) * amount                   (amount null: h' = h), in the compute type
//
// h_before is h of the request's row before, as it was before this last step: of this step's rows where the row is not
// its request's first, else what the request's state line kept (zeros in a line taken anew). A workgroup takes `chunk`
// consecutive rows in order and keeps h of the last one; for its first row it works out h of the row before once more
// (only reading: the new streams lie in memory of their own). The state line of a request is read and written by the one
// workgroup that has the request's first row of the step: it also works out h of the request's last row. So no workgroup
// waits for another, every h is computed the same way wherever it is computed, and a step of single rows is one kernel.
//
// Everything is 32-bit except what the next product reads. The order of every sum depends on the width alone.
#include "common.h"

TIS_DEFINE_LAST_ERROR(tis_hyper_streams)

typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;

struct MixArgs {
  const float* x;          // row r, stream s at x + r * ldr + s * lds (lds 0: all streams are equal)
  long ldr, lds;
  const float* y;          // [rows][ldy], or null: nothing joins
  long ldy;
  const float* y_bias;     // [D] or null
  const float* mix;        // [S][S], [from][to]
  const float* out;        // [S]
  float* x_new;            // [rows][S][D]
  const float* read;       // [S]
  const float* gain;       // [D]
  float eps;
  void* h;                 // [rows][ldh] in the compute type, or null: nothing is read
  long ldh;
  const float* amount;     // [D] or null: no row before
  float* state;            // a request's line: [D] from seq_slots[request] * state_ld
  long state_ld;
  const int* row_seq;
  const int* cu_rows;
  const int* seq_slots;
  int rows, D, S, chunk;
};

template <typename T> __device__ __forceinline__ void store4(T* p, f32x4 v);
template <> __device__ __forceinline__ void store4<float>(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
template <> __device__ __forceinline__ void store4<bf16>(bf16* p, f32x4 v) {
  bf16x4 w;
#pragma unroll
  for (int i = 0; i < 4; ++i) w[i] = static_cast<__bf16>(v[i]);
  *reinterpret_cast<bf16x4*>(p) = w;
}

// Widths in steps of 4, up to four streams: a thread owns P4 runs of four channels in every stream.
template <typename T, int S, int P4>
__global__ __launch_bounds__(1024) void mix_streams_kernel(MixArgs a) {
  __shared__ float red[16];
  const int t = threadIdx.x, nt = blockDim.x, D4 = a.D / 4;
  float mix[S][S], out[S], read[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
#pragma unroll
    for (int q = 0; q < S; ++q) mix[s][q] = a.y ? a.mix[s * S + q] : 0.f;
    out[s] = a.y ? a.out[s] : 0.f;
    read[s] = a.h ? a.read[s] : 0.f;
  }
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  // u of row r, and with `store` the row's new streams
  auto row_u = [&](long r, bool store, f32x4 (&u)[P4]) {
#pragma unroll
    for (int p = 0; p < P4; ++p) {
      const int c4 = t + p * nt;
      u[p] = zero;
      if (c4 >= D4) continue;
      const float* src = a.x + r * a.ldr + c4 * 4;
      f32x4 x[S];
#pragma unroll
      for (int s = 0; s < S; ++s) x[s] = *reinterpret_cast<const f32x4*>(src + s * a.lds);
      if (a.y) {
        f32x4 y = *reinterpret_cast<const f32x4*>(a.y + r * a.ldy + c4 * 4);
        if (a.y_bias) y += *reinterpret_cast<const f32x4*>(a.y_bias + c4 * 4);
        f32x4 n[S];
#pragma unroll
        for (int q = 0; q < S; ++q) {
          n[q] = out[q] * y;
#pragma unroll
          for (int s = 0; s < S; ++s) n[q] += mix[s][q] * x[s];
        }
#pragma unroll
        for (int q = 0; q < S; ++q) {
          x[q] = n[q];
          if (store) *reinterpret_cast<f32x4*>(a.x_new + (r * S + q) * a.D + c4 * 4) = n[q];
        }
      }
#pragma unroll
      for (int s = 0; s < S; ++s) u[p] += read[s] * x[s];
    }
  };
  // u becomes h
  auto norm = [&](f32x4 (&u)[P4]) {
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < P4; ++p) ss += u[p][0] * u[p][0] + u[p][1] * u[p][1] + u[p][2] * u[p][2] + u[p][3] * u[p][3];
    const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
#pragma unroll
    for (int p = 0; p < P4; ++p) {
      const int c4 = t + p * nt;
      if (c4 < D4) u[p] = u[p] * inv * *reinterpret_cast<const f32x4*>(a.gain + c4 * 4);
    }
  };
  const long r0 = (long)blockIdx.x * a.chunk, r1 = min(r0 + a.chunk, (long)a.rows);
  f32x4 before[P4], amount[P4];
#pragma unroll
  for (int p = 0; p < P4; ++p) {
    before[p] = zero;
    const int c4 = t + p * nt;
    amount[p] = (a.amount && c4 < D4) ? *reinterpret_cast<const f32x4*>(a.amount + c4 * 4) : zero;
  }
  for (long r = r0; r < r1; ++r) {
    f32x4 u[P4];
    row_u(r, true, u);
    if (!a.h) continue;
    norm(u);
    T* dst = static_cast<T*>(a.h) + r * a.ldh;
    if (!a.amount) {
#pragma unroll
      for (int p = 0; p < P4; ++p)
        if (t + p * nt < D4) store4<T>(dst + (t + p * nt) * 4, u[p]);
      continue;
    }
    const int seq = a.row_seq[r], first = a.cu_rows[seq], n = a.cu_rows[seq + 1] - first;
    if (r == first) {
      float* line = a.state + (long)a.seq_slots[seq] * a.state_ld;
      f32x4 kept[P4];
#pragma unroll
      for (int p = 0; p < P4; ++p)
        before[p] = t + p * nt < D4 ? *reinterpret_cast<const f32x4*>(line + (t + p * nt) * 4) : zero;
      if (n > 1) {
        row_u(first + n - 1, false, kept);
        norm(kept);
      } else {
#pragma unroll
        for (int p = 0; p < P4; ++p) kept[p] = u[p];
      }
#pragma unroll
      for (int p = 0; p < P4; ++p)
        if (t + p * nt < D4) *reinterpret_cast<f32x4*>(line + (t + p * nt) * 4) = kept[p];
    } else if (r == r0) {
      row_u(r - 1, false, before);
      norm(before);
    }
#pragma unroll
    for (int p = 0; p < P4; ++p) {
      if (t + p * nt < D4) store4<T>(dst + (t + p * nt) * 4, u[p] + (before[p] - u[p]) * amount[p]);
      before[p] = u[p];
    }
  }
}

// Any width, any number of streams: a workgroup a row, values worked out again where they are needed again.
static constexpr int MS_THREADS = 256;

template <typename T>
__global__ __launch_bounds__(MS_THREADS) void mix_streams_any_kernel(MixArgs a) {
  __shared__ float red[16];
  const long r = blockIdx.x;
  const int t = threadIdx.x;
  auto joined = [&](long row, int q, int c) {           // channel c of stream q after the mix
    if (!a.y) return a.x[row * a.ldr + q * a.lds + c];
    float v = a.out[q] * (a.y[row * a.ldy + c] + (a.y_bias ? a.y_bias[c] : 0.f));
    for (int s = 0; s < a.S; ++s) v += a.mix[s * a.S + q] * a.x[row * a.ldr + s * a.lds + c];
    return v;
  };
  auto u_at = [&](long row, int c) {
    float u = 0.f;
    for (int q = 0; q < a.S; ++q) u += a.read[q] * joined(row, q, c);
    return u;
  };
  auto inverse_rms = [&](long row) {
    float ss = 0.f;
    for (int c = t; c < a.D; c += MS_THREADS) {
      const float u = u_at(row, c);
      ss += u * u;
    }
    return 1.f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
  };
  if (a.y)
    for (int c = t; c < a.D; c += MS_THREADS)
      for (int q = 0; q < a.S; ++q) a.x_new[(r * a.S + q) * a.D + c] = joined(r, q, c);
  if (!a.h) return;
  T* dst = static_cast<T*>(a.h) + r * a.ldh;
  const float inv = inverse_rms(r);
  if (!a.amount) {
    for (int c = t; c < a.D; c += MS_THREADS) dst[c] = from_f<T>(u_at(r, c) * inv * a.gain[c]);
    return;
  }
  const int seq = a.row_seq[r], first = a.cu_rows[seq], last = a.cu_rows[seq + 1] - 1;
  float* line = a.state + (long)a.seq_slots[seq] * a.state_ld;
  const bool begins = r == first;
  const float inv_before = begins ? 0.f : inverse_rms(r - 1);
  const float inv_last = begins && last > r ? inverse_rms(last) : inv;
  for (int c = t; c < a.D; c += MS_THREADS) {
    const float g = a.gain[c], h = u_at(r, c) * inv * g;
    const float before = begins ? line[c] : u_at(r - 1, c) * inv_before * g;
    dst[c] = from_f<T>(h + (before - h) * a.amount[c]);
    if (begins) line[c] = last > r ? u_at(last, c) * inv_last * g : h;
  }
}

// x_new must not overlap x: old streams are read again for a row before, and where sizes are not the usual ones.
TIS_EXPORT int tis_mix_streams(int dtype, const float* x, long ldr, long lds, const float* y, long ldy, const float* y_bias,
                               const float* mix, const float* out, float* x_new, const float* read, const float* gain,
                               float eps, void* h, long ldh, const float* amount, float* state, long state_ld,
                               const int* row_seq, const int* cu_rows, const int* seq_slots, int rows, int D, int S,
                               int chunk, hipStream_t stream) {
  if (rows == 0) return 0;
  if (rows < 0 || D < 1 || S < 1 || S > 4096 || chunk < 1 || !x || (!y && !h))
    return tis_fail("mix_streams: bad arguments rows=%d width=%d streams=%d", rows, D, S);
  if (y && (!mix || !out || !x_new)) return tis_fail("mix_streams: a result that joins needs a mix, factors and new streams");
  if (h && (!read || !gain)) return tis_fail("mix_streams: a norm needs the streams' weights and a gain");
  if (y && x == x_new) return tis_fail("mix_streams: the new streams need memory of their own");
  if (amount && (!h || !state || !row_seq || !cu_rows || !seq_slots || state_ld < D))
    return tis_fail("mix_streams: a row before needs its norm, kept rows of %d and the rows' requests", D);
  const MixArgs a{x, ldr, lds, y, ldy, y_bias, mix, out, x_new, read, gain, eps, h, ldh, amount, state, state_ld, row_seq,
                  cu_rows, seq_slots, rows, D, S, chunk};
  if (dtype != TIS_F32 && dtype != TIS_BF16) return tis_fail("unknown dtype code %d", dtype);
  auto at16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
  const bool wide = D % 4 == 0 && D <= 16384 && S <= 4 && ldr % 4 == 0 && lds % 4 == 0 && ldy % 4 == 0 && ldh % 4 == 0 &&
                    state_ld % 4 == 0 && at16(x) && at16(y) && at16(y_bias) && at16(x_new) && at16(gain) && at16(h) &&
                    at16(amount) && at16(state);
  if (!wide) {
    if (dtype == TIS_F32) mix_streams_any_kernel<float><<<rows, MS_THREADS, 0, stream>>>(a);
    else mix_streams_any_kernel<bf16><<<rows, MS_THREADS, 0, stream>>>(a);
    return tis_launch_status("mix_streams");
  }
  const int p4 = D <= 4096 ? 1 : 4;
  const int threads = (D / 4 + p4 * TIS_WAVE - 1) / (p4 * TIS_WAVE) * TIS_WAVE;
  const int grid = (rows + chunk - 1) / chunk;
#define MS_LAUNCH(T, SV)                                                                      \
  if (p4 == 1) mix_streams_kernel<T, SV, 1><<<grid, threads, 0, stream>>>(a);                 \
  else mix_streams_kernel<T, SV, 4><<<grid, threads, 0, stream>>>(a);
#define MS_BY_STREAMS(T)            \
  if (S == 1) { MS_LAUNCH(T, 1) }   \
  else if (S == 2) { MS_LAUNCH(T, 2) } \
  else if (S == 3) { MS_LAUNCH(T, 3) } \
  else { MS_LAUNCH(T, 4) }
  if (dtype == TIS_F32) { MS_BY_STREAMS(float) }
  else { MS_BY_STREAMS(bf16) }
#undef MS_BY_STREAMS
#undef MS_LAUNCH
  return tis_launch_status("mix_streams");
}
