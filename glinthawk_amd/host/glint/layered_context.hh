// Context memory of designs whose layers keep different things per sequence: cache rows that grow with the sequence (attention) or a
// recurrent state of fixed size.  A ContextPlan lays the parts of all layer runs out in one region; a context is one such region plus
// the length of the sequence in it.  Recurrent state fixes the order of tokens: a context takes the token at its
// length next, or starts again at position 0.  Static and paged contexts as for Llama2 (Context / DynamicContext): one allocation, or
// 2 MiB blocks committed as the rows grow and dropped when the slot restarts.
#pragma once

#include <algorithm>
#include <cstddef>
#include <cstdint>
#include <memory>
#include <optional>
#include <vector>

#include "glint/types.hh"

namespace glint {

struct ContextPlan
{
  struct Part
  {
    uint64_t offset { 0 };    // from the start of the region
    uint64_t row_bytes { 0 }; // cache row of one token; 0: a state
    uint64_t bytes { 0 };
    uint32_t group { 1 };     // tokens whose rows are laid out together
    // of the part, for a sequence of `tokens` tokens
    uint64_t needed( const uint64_t tokens ) const { return row_bytes == 0 ? bytes : std::min( bytes, row_bytes * ( ( tokens + group - 1 ) / group * group ) ); }
  };
  static constexpr uint64_t ALIGN = 256;

  std::vector<Part> parts {}; // one or more per layer run, in the order a design adds them
  uint64_t bytes { 0 };
  uint32_t max_positions { 0 };

  explicit ContextPlan( uint32_t positions = 0 )
    : max_positions( positions )
  {
  }
  void add_rows( const uint64_t row_bytes, const uint32_t group = 1 )
  {
    add( row_bytes, row_bytes * ( ( (uint64_t)max_positions + group - 1 ) / group * group ), group );
  }
  void add_state( const uint64_t state_bytes ) { add( 0, state_bytes, 1 ); }

private:
  void add( const uint64_t row_bytes, const uint64_t n, const uint32_t group )
  {
    parts.push_back( { bytes, row_bytes, n, group } );
    bytes += ( n + ALIGN - 1 ) / ALIGN * ALIGN;
  }
};

// settings of a node that hosts a whole run-time sized model: what the context manager, the contexts and the driver read
struct DesignSettings
{
  std::shared_ptr<const ContextPlan> plan {};
  uint64_t concurrency_limit { 1 };
  uint64_t max_context_count { 1 };
  bool randomize_parameters { false };
};

class LayeredContext
{
  void* base_ { nullptr };
  uint32_t length_ { 0 };

public:
  void* data() const { return base_; }
  bool empty() const { return base_ == nullptr; }
  uint32_t length() const { return length_; }
  // whether tokens may be appended from `pos` on
  bool takes( const uint32_t pos ) const { return empty() || pos == 0 || pos == length_; }
  void set_length( const uint32_t n ) { length_ = n; }
  // static contexts have nothing to commit
  bool prepare( uint32_t, uint32_t ) { return true; }

protected:
  LayeredContext() = default;
  void set_base( void* p ) { base_ = p; }
};

template<typename VirtualMemoryRegion>
class DynamicLayeredContext : public LayeredContext
{
  std::shared_ptr<const ContextPlan> plan_ {};
  std::optional<VirtualMemoryRegion> storage_ {};
  std::vector<bool> committed_ {};
  size_t blocks_committed_ { 0 };
  size_t clears_ { 0 };

public:
  static constexpr size_t BLOCK_SIZE = 2 * 1024 * 1024;

  explicit DynamicLayeredContext( const DesignSettings& settings, const bool make_empty = false )
    : plan_( settings.plan )
  {
    if ( !make_empty ) {
      const uint64_t blocks = ( plan_->bytes + BLOCK_SIZE - 1 ) / BLOCK_SIZE;
      storage_.emplace( blocks * BLOCK_SIZE );
      committed_.resize( blocks, false );
      set_base( storage_->ptr() );
    }
  }

  // commits what `n_tokens` tokens from `pos` on need; a sequence that starts again drops what the last one had
  bool prepare( const uint32_t pos, const uint32_t n_tokens )
  {
    if ( empty() ) {
      return true;
    }
    if ( pos == 0 && blocks_committed_ > 0 ) {
      storage_->clear();
      std::fill( committed_.begin(), committed_.end(), false );
      blocks_committed_ = 0;
      clears_++;
    }
    for ( const auto& part : plan_->parts ) {
      const uint64_t need = part.needed( (uint64_t)pos + n_tokens );
      if ( need == 0 ) {
        continue;
      }
      for ( uint64_t b = part.offset / BLOCK_SIZE; b <= ( part.offset + need - 1 ) / BLOCK_SIZE; b++ ) {
        if ( !committed_[b] ) {
          storage_->allocate_span( static_cast<const uint8_t*>( storage_->ptr() ) + b * BLOCK_SIZE, BLOCK_SIZE );
          committed_[b] = true;
          blocks_committed_++;
        }
      }
    }
    return true;
  }

  size_t blocks_committed() const { return blocks_committed_; }
  size_t clears() const { return clears_; }
};

} // namespace glint
