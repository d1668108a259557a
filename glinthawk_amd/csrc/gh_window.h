// Shapes and addresses of the windowed attention (gh_attn_window.hip) and of what writes its cache rows.
#pragma once

#include "gh_common.h"

namespace gh {

struct WindowShape
{
  uint32_t heads, kv_heads, group; // query heads, kv heads, query heads per kv head
  uint32_t dim, vdim, dpad, vpad;  // padded head sizes of the cache
  uint32_t window, keep_first, n_dist;
  float scale;
  bool values_are_keys; // a head is in the cache once; the keys' factors lie beside
  __host__ __device__ uint32_t k_elems() const { return kv_heads * dpad; }
  __host__ __device__ uint32_t row_elems() const { return kv_heads * ( values_are_keys ? dpad : dpad + vpad ); }
};

struct WindowRows
{
  void* const* rows; // context regions; NULL: no context
  uint64_t offset;   // bytes from there to this layer's rows
  uint64_t factors;  // and to its key factors
  const uint32_t* start_pos;
  uint32_t n_tokens;
};

// Key factors: GH_WINDOW_FACTOR_GROUP tokens of a kv head side by side, so that a head's factors of neighbouring keys come in one line.
__device__ __forceinline__ uint64_t factor_index( uint32_t key, uint32_t kv_head, uint32_t kv_heads )
{
  return ( (uint64_t)( key / GH_WINDOW_FACTOR_GROUP ) * kv_heads + kv_head ) * GH_WINDOW_FACTOR_GROUP + key % GH_WINDOW_FACTOR_GROUP;
}

inline WindowShape window_shape( const gh_window_attn* a )
{
  WindowShape s;
  s.heads = a->heads;
  s.kv_heads = a->kv_heads;
  s.group = a->kv_heads ? a->heads / a->kv_heads : 0;
  s.dim = a->dim;
  s.vdim = a->vdim;
  s.dpad = ( a->dim + 7 ) / 8 * 8;
  s.vpad = ( a->vdim + 7 ) / 8 * 8;
  s.window = a->window ? a->window : 0xffffffffu;
  s.keep_first = a->keep_first;
  s.n_dist = a->n_dist ? a->n_dist : 1;
  s.scale = a->scale;
  s.values_are_keys = a->values_are_keys != 0;
  return s;
}

inline bool window_shape_ok( const gh_window_attn* a )
{
  return a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->dim > 0 && a->vdim > 0 && a->dim <= 512 && a->vdim <= 512 && a->heads <= 4096
         && ( !a->values_are_keys || a->dim == a->vdim );
}

} // namespace gh
